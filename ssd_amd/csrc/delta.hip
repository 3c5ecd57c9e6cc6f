// Gated delta rule over a recurrent fp32 state (linear attention whose write corrects what the state already answers to the key):
//     S <- g_t S;   u = beta_t (v_t - S^T k_t);   S <- S + k_t u^T;   o_t = S^T q_t        (S: [D][Dv] per sequence and head, S = 0 first)
// g_t is one number per head, or one per head and key channel (it scales the rows of S).  q / k heads may be shared by several heads.
//  * ssd_delta_prep   from fp32 projection rows: short causal convolution + silu on every channel of q, k and v; q and k made unit vectors
//                     per head, x / sqrt(sum x^2 + 1e-6), q also times D^-0.5; <q, k>; beta = sigmoid(.); the per-head decay
//                     exp(-rate_h softplus(. + bias_h)) when it is one number per head; and (optional) element-type copies of some columns
//                     (the inner rows of low-rank projections, as the next product's input)
//  * ssd_delta_scan   the recurrence over a portion's rows; also saves the slot's last taps - 1 convolution inputs
// Layout: a head's key channels are padded to DP (32, or a multiple of 64 up to 512) zeros: qk rows [T][G][2][DP] (q, then k), decay rows
// [.. H][DP], state [slots][H][Dv][DP] -- TRANSPOSED, a value column's key channels contiguous.  A value column of S depends on the other
// columns only through k, q, g and beta, so P = 8 or 16 lanes own a column (DP / P channels each, in registers) and the two sums over the
// key channels -- S^T k and S^T q, both of the DECAYED state: o = (g S)^T q + u <q, k>, the read-out of the updated state -- meet by DPP
// adds inside the wave: no barrier between tokens.  Rows are staged through LDS TB at a time, the next batch travels in registers
// meanwhile.  The arithmetic of a row does not depend on how a prompt is cut nor on the batch: one chain per state element in token
// order, sums in a fixed order.
#include "common.h"
#include "shortconv.h"

namespace {

template <typename T> __device__ __forceinline__ void stf(T* p, float v);
template <> __device__ __forceinline__ void stf<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void stf<bf16_t>(bf16_t* p, float v) { *p = (bf16_t)f2bf(v); }

__device__ __forceinline__ float siluf_(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float sigmoidf_(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplusf_(float z) { return z > 20.0f ? z : log1pf(expf(z)); }

constexpr int MAX_D = 512;

struct PrepArgs {
  const float* proj; long ld; int col_off; int conv_c0; const float* conv_state; int C; int taps;
  int b_off, a_off; const float* rate; const float* bias; int lr_off, lr_n; long ld_lr;
};

// grid = (tokens, column blocks); the work of a token is a list of wave units: one per q / k head (both vectors, their norms, their
// product, the scalars of the heads that share them), one per 64 value channels, one per 64 copied columns.
template <typename T, int TAPS>
__global__ void __launch_bounds__(256)
delta_prep_kernel(PrepArgs a, const T* __restrict__ cw, const int64_t* __restrict__ positions, const int32_t* __restrict__ cu_q,
                  int q_per_seq, const int32_t* __restrict__ state_slots, int B, float* __restrict__ qk, float* __restrict__ vrows,
                  float4* __restrict__ scalars, T* __restrict__ lr_out, int H, int G, int D, int Dv, int DP) {
  constexpr int KEEP = MAX_D / 64;
  const int t = blockIdx.x, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int b = seq_of_row(cu_q, q_per_seq, B, t);
  const int row0 = cu_q ? cu_q[b] : b * q_per_seq;
  const long p0 = positions[row0];
  const float* st = a.conv_state + (size_t)state_slots[b] * (a.taps - 1) * a.C;
  auto val = [&](int c) {
    return siluf_(conv_at<T, TAPS>(a.proj, a.ld, (long)a.col_off + c, a.conv_c0 + c, a.C, cw + (size_t)c * a.taps, a.taps, st, t, row0, p0, 0.f));
  };
  const int R = H / G, Nk = G * D, Nv = H * Dv;
  const int v_units = (Nv + 63) >> 6, lr_units = lr_out ? (int)((a.ld_lr + 63) >> 6) : 0;
  const float* row = a.proj + (size_t)t * a.ld;
  for (int u = blockIdx.y * 4 + wave; u < G + v_units + lr_units; u += 4 * gridDim.y) {
    if (u < G) {
      float vq[KEEP], vk[KEEP], sq = 0.f, sk = 0.f, dot = 0.f;
#pragma unroll
      for (int i = 0; i < KEEP; ++i) {
        vq[i] = vk[i] = 0.f;
        const int d = lane + i * 64;
        if (i * 64 < D && d < D) { vq[i] = val(u * D + d); vk[i] = val(Nk + u * D + d); }
        sq = fmaf(vq[i], vq[i], sq);
        sk = fmaf(vk[i], vk[i], sk);
        dot = fmaf(vq[i], vk[i], dot);
      }
      sq = wave_sum(sq); sk = wave_sum(sk); dot = wave_sum(dot);
      const float rq = 1.0f / sqrtf(sq + 1e-6f) / sqrtf((float)D), rk = 1.0f / sqrtf(sk + 1e-6f);
      float* dst = qk + ((size_t)t * G + u) * 2 * DP;
#pragma unroll
      for (int i = 0; i < KEEP; ++i) {
        const int d = lane + i * 64;
        if (d < DP) { dst[d] = vq[i] * rq; dst[DP + d] = vk[i] * rk; }
      }
      for (int j = lane; j < R; j += 64) {
        const int h = u * R + j;
        const float g = a.a_off >= 0 ? expf(-a.rate[h] * softplusf_(row[a.a_off + h] + a.bias[h])) : 1.0f;
        scalars[(size_t)t * H + h] = float4{sigmoidf_(row[a.b_off + h]), g, dot * rq * rk, 0.f};
      }
    } else if (u < G + v_units) {
      const int c = (u - G) * 64 + lane;
      if (c < Nv) vrows[(size_t)t * Nv + c] = val(2 * Nk + c);
    } else {
      const int c = (u - G - v_units) * 64 + lane;
      if (c < a.ld_lr) stf<T>(lr_out + (size_t)t * a.ld_lr + c, c < a.lr_n ? row[a.lr_off + c] : 0.f);
    }
  }
}

struct ConvSave { const float* proj; long ld; int off, C; float* state; int taps; };

template <int P, int NJ, int TB, bool CH>
__global__ void __launch_bounds__(256)
delta_scan_kernel(const float4* __restrict__ qk, const float* __restrict__ vrows, const float4* __restrict__ scalars,
                  const float4* __restrict__ decay, long ldd4, const int64_t* __restrict__ positions, const int32_t* __restrict__ cu_q,
                  int q_per_seq, const int32_t* __restrict__ state_slots, float* __restrict__ state, float* __restrict__ out, int H, int G,
                  int Dv, ConvSave cs) {
  constexpr int D4 = P * NJ, COLS = 256 / P;               // float4 per head vector, value columns per workgroup
  constexpr int F4 = (TB * D4 + 255) / 256, FV = (TB * COLS + 255) / 256;
  __shared__ float4 sk[TB * D4], sq[TB * D4], sg[CH ? TB * D4 : 1], ss[TB];
  __shared__ float sv[TB * COLS], so[TB * COLS];
  const int b = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * COLS, tid = threadIdx.x;
  const int col = tid / P, p = tid % P, e = c0 + col;
  const int grp = h / (H / G);
  const int row0 = cu_q ? cu_q[b] : b * q_per_seq;
  const int row1 = cu_q ? cu_q[b + 1] : (b + 1) * q_per_seq;
  if (row1 <= row0) return;
  const int slot = state_slots[b];
  const long p0 = positions[row0];
  float4* sp = reinterpret_cast<float4*>(state) + (((size_t)slot * H + h) * Dv + e) * D4 + p;
  float4 s[NJ];
#pragma unroll
  for (int j = 0; j < NJ; ++j) s[j] = (p0 == 0 || e >= Dv) ? float4{0.f, 0.f, 0.f, 0.f} : sp[P * j];

  float4 rk[F4], rq[F4], rg[F4], rs;
  float rv[FV];
  auto fetch = [&](int r) {
    const int nb = min(row1 - r, TB);
#pragma unroll
    for (int f = 0; f < F4; ++f) {
      const int i = tid + 256 * f, tt = i / D4, d = i % D4;
      rq[f] = rk[f] = rg[f] = float4{0.f, 0.f, 0.f, 0.f};
      if (tt < nb) {
        const float4* src = qk + ((size_t)(r + tt) * G + grp) * 2 * D4 + d;
        rq[f] = src[0];
        rk[f] = src[D4];
        if (CH) rg[f] = decay[(size_t)(r + tt) * ldd4 + h * D4 + d];
      }
    }
#pragma unroll
    for (int f = 0; f < FV; ++f) {
      const int i = tid + 256 * f, tt = i / COLS, c = c0 + i % COLS;
      rv[f] = tt < nb && c < Dv ? vrows[((size_t)(r + tt) * H + h) * Dv + c] : 0.f;
    }
    if (tid < nb) rs = scalars[(size_t)(r + tid) * H + h];
  };
  auto put_out = [&](int r, int nb) {
#pragma unroll
    for (int f = 0; f < FV; ++f) {
      const int i = tid + 256 * f, tt = i / COLS, c = c0 + i % COLS;
      if (i < TB * COLS && tt < nb && c < Dv) out[((size_t)(r + tt) * H + h) * Dv + c] = so[i];
    }
  };
  fetch(row0);
  for (int r = row0; r < row1; r += TB) {
    const int nb = min(row1 - r, TB);
    __syncthreads();                      // the previous batch is walked: its staged rows are free, its outputs are in LDS
    if (r > row0) put_out(r - TB, TB);
#pragma unroll
    for (int f = 0; f < F4; ++f) {
      const int i = tid + 256 * f;
      if (i < TB * D4) {
        sq[i] = rq[f];
        sk[i] = rk[f];
        if (CH) sg[i] = rg[f];
      }
    }
#pragma unroll
    for (int f = 0; f < FV; ++f)
      if (tid + 256 * f < TB * COLS) sv[tid + 256 * f] = rv[f];
    if (tid < nb) ss[tid] = rs;
    __syncthreads();
    if (r + TB < row1) fetch(r + TB);
    // the staged values of a token are read one token ahead of their use: the LDS latency hides behind the current token's chain
    float4 k[NJ], q[NJ], g[NJ], sc;
    float v;
    auto read = [&](int tt) {
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        const int i = tt * D4 + P * j + p;
        k[j] = sk[i];
        q[j] = sq[i];
        if (CH) g[j] = sg[i];
      }
      sc = ss[tt];                        // beta, decay of the head, <q, k>
      v = sv[tt * COLS + col];
    };
    auto step = [&](int tt) {
      float4 kc[NJ];
      const float beta = sc.x, gh = sc.y, kq = sc.z, vc = v;
      float4 ak{0.f, 0.f, 0.f, 0.f}, aq{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        kc[j] = k[j];
        const float4 gj = CH ? g[j] : float4{gh, gh, gh, gh};
        s[j].x *= gj.x; s[j].y *= gj.y; s[j].z *= gj.z; s[j].w *= gj.w;
        ak.x = fmaf(s[j].x, k[j].x, ak.x); ak.y = fmaf(s[j].y, k[j].y, ak.y);
        ak.z = fmaf(s[j].z, k[j].z, ak.z); ak.w = fmaf(s[j].w, k[j].w, ak.w);
        aq.x = fmaf(s[j].x, q[j].x, aq.x); aq.y = fmaf(s[j].y, q[j].y, aq.y);
        aq.z = fmaf(s[j].z, q[j].z, aq.z); aq.w = fmaf(s[j].w, q[j].w, aq.w);
      }
      read(min(tt + 1, TB - 1));
      const float dk = col_sum<P>((ak.x + ak.y) + (ak.z + ak.w));
      const float dq = col_sum<P>((aq.x + aq.y) + (aq.z + aq.w));
      const float u = beta * (vc - dk);
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        s[j].x = fmaf(kc[j].x, u, s[j].x); s[j].y = fmaf(kc[j].y, u, s[j].y);
        s[j].z = fmaf(kc[j].z, u, s[j].z); s[j].w = fmaf(kc[j].w, u, s[j].w);
      }
      if (p == 0) so[tt * COLS + col] = fmaf(u, kq, dq);
    };
    read(0);
    if (nb == TB) {
#pragma unroll 4
      for (int tt = 0; tt < TB; ++tt) step(tt);
    } else {
      for (int tt = 0; tt < nb; ++tt) step(tt);
    }
  }
  __syncthreads();
  {
    const int last = row0 + (row1 - row0 - 1) / TB * TB;
    put_out(last, row1 - last);
  }
  if (e < Dv) {
#pragma unroll
    for (int j = 0; j < NJ; ++j) sp[P * j] = s[j];
  }
  if (cs.taps > 1) {           // the slot's saved convolution inputs: every workgroup of the sequence saves its share of the channels
    const int wg = h * gridDim.z + blockIdx.z, nwg = H * gridDim.z, chunk = (cs.C + nwg - 1) / nwg;
    save_conv_state(cs.proj, cs.ld, cs.off, cs.C, cs.state, cs.taps, slot, row0, row1, p0, wg * chunk, min(cs.C, (wg + 1) * chunk));
  }
}

bool dp_ok(int D, int DP) { return D > 0 && D <= MAX_D && DP == (D <= 32 ? 32 : (D + 63) / 64 * 64); }

}  // namespace

#define LAUNCH_OK() (hipGetLastError() == hipSuccess ? SSD_OK : SSD_ERR_LAUNCH)

extern "C" int ssd_delta_prep(const void* proj_rows, long ld, int col_off, const void* conv_w, int taps, const float* conv_state, int C,
                              int conv_c0, const int32_t* state_slots, const int64_t* positions, const int32_t* cu_q, int q_per_seq, int B,
                              int b_off, int a_off, const float* rate, const float* bias, int lr_off, int lr_n, void* lr_out, long ld_lr,
                              void* qk_rows, void* v_rows, void* scalars, int T, int H, int G, int D, int Dv, int DP, int f32,
                              void* stream) {
  if (!proj_rows || !conv_w || !conv_state || !state_slots || !positions || !qk_rows || !v_rows || !scalars ||
      (a_off >= 0 && (!rate || !bias)))
    return SSD_ERR_ARG;
  const long n = 2L * G * D + (long)H * Dv;
  if (T <= 0 || B <= 0 || H <= 0 || G <= 0 || H % G || Dv <= 0 || !dp_ok(D, DP) || taps < 1 || taps > CONV_MAX_TAPS ||
      (!cu_q && q_per_seq <= 0) || col_off < 0 || conv_c0 < 0 || C < conv_c0 + n || ld < col_off + n || b_off < 0 || ld < (long)b_off + H ||
      (a_off >= 0 && ld < (long)a_off + H) || (lr_out && (lr_off < 0 || lr_n <= 0 || ld_lr < lr_n || ld < (long)lr_off + lr_n)))
    return SSD_ERR_SHAPE;
  const PrepArgs a{(const float*)proj_rows, ld, col_off, conv_c0, conv_state, C, taps, b_off, a_off, rate, bias, lr_off, lr_n, ld_lr};
  const int units = G + (H * Dv + 63) / 64 + (lr_out ? (int)((ld_lr + 63) / 64) : 0), ub = (units + 3) / 4;
  const dim3 grid(T, T >= 256 ? (ub < 4 ? ub : 4) : (ub < 64 ? ub : 64));
#define PREP(TY, TAPS)                                                                                                              \
  hipLaunchKernelGGL((delta_prep_kernel<TY, TAPS>), grid, dim3(256), 0, (hipStream_t)stream, a, (const TY*)conv_w, positions, cu_q,    \
                     q_per_seq, state_slots, B, (float*)qk_rows, (float*)v_rows, (float4*)scalars, (TY*)lr_out, H, G, D, Dv, DP)
#define PREP_T(TAPS) do { if (f32) PREP(float, TAPS); else PREP(bf16_t, TAPS); } while (0)
  CONV_TAPS(taps, PREP_T);
#undef PREP_T
#undef PREP
  return LAUNCH_OK();
}

extern "C" int ssd_delta_scan(const void* qk_rows, const void* v_rows, const void* scalars, const float* decay_rows, long ldd,
                              const int64_t* positions, const int32_t* cu_q, int q_per_seq, const int32_t* state_slots, void* state,
                              void* out_rows, int B, int H, int G, int D, int Dv, int DP, const void* proj_rows, long ld, int conv_off, int C,
                              void* conv_state, int taps, void* stream) {
  if (!qk_rows || !v_rows || !scalars || !positions || !state_slots || !state || !out_rows) return SSD_ERR_ARG;
  if (taps > 1 && (!proj_rows || !conv_state)) return SSD_ERR_ARG;
  if (B <= 0 || H <= 0 || G <= 0 || H % G || H > 65535 || Dv <= 0 || !dp_ok(D, DP) || (!cu_q && q_per_seq <= 0) || taps < 1 ||
      taps > CONV_MAX_TAPS || (taps > 1 && (C <= 0 || conv_off < 0 || ld < (long)conv_off + C)))
    return SSD_ERR_SHAPE;
  if (((uintptr_t)qk_rows | (uintptr_t)scalars | (uintptr_t)state | (uintptr_t)decay_rows) % 16 ||
      (decay_rows && (ldd % 4 || ldd < (long)H * DP)))
    return SSD_ERR_SHAPE;
  const ConvSave cs{(const float*)proj_rows, ld, conv_off, C, (float*)conv_state, taps};
  const int cols = DP == 32 ? 32 : 16, zb = (Dv + cols - 1) / cols;
  if (zb > 65535) return SSD_ERR_SHAPE;
  const dim3 grid(B, H, zb);
#define DELTA(P, NJ, TB, CH)                                                                                                              \
  hipLaunchKernelGGL((delta_scan_kernel<P, NJ, TB, CH>), grid, dim3(256), 0, (hipStream_t)stream, (const float4*)qk_rows,                 \
                     (const float*)v_rows, (const float4*)scalars, (const float4*)decay_rows, ldd / 4, positions, cu_q, q_per_seq,        \
                     state_slots, (float*)state, (float*)out_rows, H, G, Dv, cs)
#define DELTA2(P, NJ, TB) do { if (decay_rows) DELTA(P, NJ, TB, true); else DELTA(P, NJ, TB, false); } while (0)
  switch (DP) {
    case 32: DELTA2(8, 1, 16); break;
    case 64: DELTA2(16, 1, 16); break;
    case 128: DELTA2(16, 2, 16); break;
    case 192: DELTA2(16, 3, 16); break;
    case 256: DELTA2(16, 4, 16); break;
    case 320: DELTA2(16, 5, 8); break;
    case 384: DELTA2(16, 6, 8); break;
    case 448: DELTA2(16, 7, 8); break;
    default: DELTA2(16, 8, 8); break;
  }
#undef DELTA2
#undef DELTA
  return LAUNCH_OK();
}
