// Linear attention over a recurrent fp32 outer-product memory with one decay per head and token:
//     S_t = a_t S_(t-1) + b_t k_t v_t^T,   o_t = c S_t^T q_t            (S: [D][Dv] per sequence and head, S = 0 before position 0)
// in two kinds:
//   fixed decay        a_t = decay_h, b_t = 1 (retention)
//   exponential gates  from two projected numbers per head and token: log input gate i = cap tanh((z_i + bias_i) / cap), log forget gate
//                      f = log sigmoid(cap tanh((z_f + bias_f) / cap)); with a running maximum m (m = 0 first) m_t = max(f + m_(t-1), i),
//                      a_t = exp(f + m_(t-1) - m_t), b_t = exp(i - m_t); and a normaliser n_t = a_t n_(t-1) + b_t k_t that divides the
//                      output: den_t = max(|c <n_t, q_t>|, exp(-m_t)) + 1e-6.  The normaliser is column Dv of S, the one whose value is 1.
//  * ssd_memory_scan    the recurrence over a portion's rows: o (undivided) [T][H * Dv] and den [T][H]; state and m written back
//  * ssd_memory_gates   (a, b, exp(-m)) of every row of a portion ahead of the scan, and m: for portions of many rows, where a batch's gates
//                       would otherwise be computed by every workgroup of the scan.  The same function, the same bits.
// The state is TRANSPOSED, state[slots][H][columns][DP]: a column's key channels contiguous, padded with zeros to DP (32, or a multiple of
// 64 up to 512).  A column of S depends on the others only through k, q and the gates: P = 8 or 16 lanes own one (DP / P channels each, in
// registers), 16 or 32 columns per workgroup, and the read-out's sum over the channels is a few DPP adds inside the wave.  Rows are staged
// through LDS TB at a time, the next batch travels in registers meanwhile; no barrier between tokens.  The arithmetic of a row does not
// depend on how a prompt is cut nor on the batch: one chain per state element in token order, sums in a fixed order.
#include "common.h"

namespace {

constexpr int MAX_D = 512;
constexpr int MODE_GATES = 0, MODE_INLINE = 1, MODE_DECAY = 2;

struct Gating { const float* bias_i; const float* bias_f; float cap; int i_off, f_off; };

__device__ __forceinline__ float log_sigmoid_(float y) { return fminf(y, 0.f) - log1pf(expf(-fabsf(y))); }

// Lane t of a wave holds the gate projections of token t (t < n <= N); m is the running maximum before token 0 and becomes the one after
// token n - 1.  Returns (a, b, exp(-m_t), 0) of the lane's token.
template <int N>
__device__ __forceinline__ float4 gate_chain(float zi, float zf, float cap, int n, float& m) {
  const int lane = threadIdx.x & 63;
  const float li = cap * tanhf(zi / cap), lf = log_sigmoid_(cap * tanhf(zf / cap));
  float mine_x = 0.f, mine_m = 0.f;
  auto link = [&](int t) {
    const float f = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(lf), t));
    const float i = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(li), t));
    const float x = f + m;
    m = fmaxf(x, i);
    mine_x = lane == t ? x : mine_x;
    mine_m = lane == t ? m : mine_m;
  };
  if (n == N) {
#pragma unroll
    for (int t = 0; t < N; ++t) link(t);
  } else {
    for (int t = 0; t < n; ++t) link(t);
  }
  return float4{expf(mine_x - mine_m), expf(li - mine_m), expf(-mine_m), 0.f};
}

__global__ void __launch_bounds__(64)
memory_gates_kernel(const float* __restrict__ proj, long ld, Gating gt, const int64_t* __restrict__ positions,
                    const int32_t* __restrict__ cu_q, int q_per_seq, const int32_t* __restrict__ state_slots, float* __restrict__ m_state,
                    float4* __restrict__ gates, int H, int copies, int ld_m) {
  const int b = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const int row0 = cu_q ? cu_q[b] : b * q_per_seq;
  const int row1 = cu_q ? cu_q[b + 1] : (b + 1) * q_per_seq;
  if (row1 <= row0) return;
  float* ms = m_state + ((size_t)state_slots[b] * H + h) * ld_m;
  float m = positions[row0] == 0 ? 0.f : ms[0];
  const float bi = gt.bias_i[h], bf = gt.bias_f[h];
  float zi = 0.f, zf = 0.f;
  auto fetch = [&](int r) {
    const int row = r + lane < row1 ? r + lane : row1 - 1;
    zi = proj[(size_t)row * ld + gt.i_off + h] + bi;
    zf = proj[(size_t)row * ld + gt.f_off + h] + bf;
  };
  fetch(row0);
  for (int r = row0; r < row1; r += 64) {
    const int n = min(row1 - r, 64);
    const float ci = zi, cf = zf;
    if (r + 64 < row1) fetch(r + 64);
    const float4 g = gate_chain<64>(ci, cf, gt.cap, n, m);
    if (lane < n) gates[(size_t)(r + lane) * H + h] = g;
  }
  for (int c = lane; c < copies; c += 64) ms[c] = m;
}

struct Rows { const float* proj; long ld; int q_off, k_off, v_off; float q_scale; };

// grid = (sequences, heads, column blocks)
template <int P, int NJ, int TB, int MODE>
__global__ void __launch_bounds__(256)
memory_scan_kernel(Rows in, const float* __restrict__ decay, const float4* __restrict__ gates, Gating gt,
                   const int64_t* __restrict__ positions, const int32_t* __restrict__ cu_q, int q_per_seq,
                   const int32_t* __restrict__ state_slots, float* __restrict__ state, float* __restrict__ m_state, int ld_m,
                   float* __restrict__ out, float* __restrict__ den, int H, int D, int Dv) {
  constexpr int D4 = P * NJ, DP = 4 * D4, COLS = 256 / P;      // float4 per key vector, padded channels, columns per workgroup
  constexpr int F = (TB * DP + 255) / 256, FV = (TB * COLS + 255) / 256;
  __shared__ float4 sk[TB * D4], sq[TB * D4], ss[TB];
  __shared__ float sv[TB * COLS], so[TB * COLS];
  const int b = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * COLS, tid = threadIdx.x;
  const int col = tid / P, p = tid % P, e = c0 + col;
  const int NC = MODE == MODE_DECAY ? Dv : Dv + 1;
  const int row0 = cu_q ? cu_q[b] : b * q_per_seq;
  const int row1 = cu_q ? cu_q[b + 1] : (b + 1) * q_per_seq;
  if (row1 <= row0) return;
  const int slot = state_slots[b];
  const bool fresh = positions[row0] == 0;
  float4* sp = reinterpret_cast<float4*>(state) + (((size_t)slot * H + h) * NC + e) * D4 + p;
  float4 s[NJ];
#pragma unroll
  for (int j = 0; j < NJ; ++j) s[j] = (fresh || e >= NC) ? float4{0.f, 0.f, 0.f, 0.f} : sp[P * j];
  float* mp = MODE == MODE_INLINE ? m_state + ((size_t)slot * H + h) * ld_m + blockIdx.z : nullptr;
  float m = MODE == MODE_INLINE && !fresh ? *mp : 0.f;          // every column block keeps a copy: none reads what another one writes
  const float fixed = MODE == MODE_DECAY ? decay[h] : 0.f;
  const float bi = MODE == MODE_INLINE ? gt.bias_i[h] : 0.f, bf = MODE == MODE_INLINE ? gt.bias_f[h] : 0.f;

  float rk[F], rq[F], rv[FV], zi = 0.f, zf = 0.f;
  float4 rg = float4{0.f, 0.f, 0.f, 0.f};
  auto fetch = [&](int r) {
    const int nb = min(row1 - r, TB);
#pragma unroll
    for (int f = 0; f < F; ++f) {
      const int i = tid + 256 * f, tt = i / DP, d = i % DP;
      rq[f] = rk[f] = 0.f;
      if (tt < nb && d < D) {
        const float* src = in.proj + (size_t)(r + tt) * in.ld + h * D + d;
        rq[f] = src[in.q_off];
        rk[f] = src[in.k_off];
      }
    }
#pragma unroll
    for (int f = 0; f < FV; ++f) {
      const int i = tid + 256 * f, tt = i / COLS, c = c0 + i % COLS;
      rv[f] = c == Dv ? 1.f : 0.f;                              // (past the last column: a column of zeros that is never written)
      if (tt < nb && c < Dv) rv[f] = in.proj[(size_t)(r + tt) * in.ld + in.v_off + h * Dv + c];
    }
    if (tid < nb) {
      if (MODE == MODE_GATES) rg = gates[(size_t)(r + tid) * H + h];
      if (MODE == MODE_INLINE) {
        zi = in.proj[(size_t)(r + tid) * in.ld + gt.i_off + h] + bi;
        zf = in.proj[(size_t)(r + tid) * in.ld + gt.f_off + h] + bf;
      }
    }
  };
  auto put_out = [&](int r, int nb) {
#pragma unroll
    for (int f = 0; f < FV; ++f) {
      const int i = tid + 256 * f, tt = i / COLS, c = c0 + i % COLS;
      if (i >= TB * COLS || tt >= nb) continue;
      if (c < Dv) out[((size_t)(r + tt) * H + h) * Dv + c] = so[i];
      else if (MODE != MODE_DECAY && c == Dv) den[(size_t)(r + tt) * H + h] = so[i];
    }
  };
  fetch(row0);
  for (int r = row0; r < row1; r += TB) {
    const int nb = min(row1 - r, TB);
    __syncthreads();                      // the previous batch is walked: its staged rows are free, its outputs are in LDS
    if (r > row0) put_out(r - TB, TB);
#pragma unroll
    for (int f = 0; f < F; ++f) {
      const int i = tid + 256 * f;
      if (i < TB * DP) {
        reinterpret_cast<float*>(sq)[i] = rq[f];
        reinterpret_cast<float*>(sk)[i] = rk[f];
      }
    }
#pragma unroll
    for (int f = 0; f < FV; ++f)
      if (tid + 256 * f < TB * COLS) sv[tid + 256 * f] = rv[f];
    if (MODE == MODE_INLINE && tid < 64) rg = gate_chain<TB>(zi, zf, gt.cap, nb, m);
    if (MODE != MODE_DECAY && tid < nb) ss[tid] = rg;
    __syncthreads();
    if (r + TB < row1) fetch(r + TB);
    // the staged values of a token are read one token ahead of their use: the LDS latency hides behind the current token's arithmetic
    float4 k[NJ], q[NJ], sc;
    float v;
    auto read = [&](int tt) {
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        k[j] = sk[tt * D4 + P * j + p];
        q[j] = sq[tt * D4 + P * j + p];
      }
      if (MODE != MODE_DECAY) sc = ss[tt];
      v = sv[tt * COLS + col];
    };
    auto step = [&](int tt) {
      const float a = MODE == MODE_DECAY ? fixed : sc.x, w = MODE == MODE_DECAY ? v : v * sc.y, floor_ = MODE == MODE_DECAY ? 0.f : sc.z;
      float4 o{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        s[j].x = fmaf(a, s[j].x, k[j].x * w); s[j].y = fmaf(a, s[j].y, k[j].y * w);
        s[j].z = fmaf(a, s[j].z, k[j].z * w); s[j].w = fmaf(a, s[j].w, k[j].w * w);
        o.x = fmaf(s[j].x, q[j].x, o.x); o.y = fmaf(s[j].y, q[j].y, o.y);
        o.z = fmaf(s[j].z, q[j].z, o.z); o.w = fmaf(s[j].w, q[j].w, o.w);
      }
      read(min(tt + 1, TB - 1));
      float y = col_sum<P>((o.x + o.y) + (o.z + o.w)) * in.q_scale;
      if (MODE != MODE_DECAY && e == Dv) y = fmaxf(fabsf(y), floor_) + 1e-6f;
      if (p == 0) so[tt * COLS + col] = y;
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
  if (e < NC) {
#pragma unroll
    for (int j = 0; j < NJ; ++j) sp[P * j] = s[j];
  }
  if (MODE == MODE_INLINE && tid == 0) *mp = m;
}

bool dp_ok(int D, int DP) { return D > 0 && D <= MAX_D && DP == (D <= 32 ? 32 : (D + 63) / 64 * 64); }
int col_blocks_of(int DP, int columns) { const int cols = DP == 32 ? 32 : 16; return (columns + cols - 1) / cols; }

}  // namespace

#define LAUNCH_OK() (hipGetLastError() == hipSuccess ? SSD_OK : SSD_ERR_LAUNCH)

extern "C" int ssd_memory_gates(const void* proj_rows, long ld, int i_off, int f_off, const float* bias_i, const float* bias_f, float cap,
                                const int64_t* positions, const int32_t* cu_q, int q_per_seq, const int32_t* state_slots, void* m_state,
                                void* gates, int B, int H, int Dv, void* stream) {
  if (!proj_rows || !bias_i || !bias_f || !positions || !state_slots || !m_state || !gates) return SSD_ERR_ARG;
  if (B <= 0 || H <= 0 || H > 65535 || Dv <= 0 || !(cap > 0.f) || i_off < 0 || f_off < 0 || ld < (long)i_off + H || ld < (long)f_off + H ||
      (!cu_q && q_per_seq <= 0) || (uintptr_t)gates % 16)
    return SSD_ERR_SHAPE;
  hipLaunchKernelGGL(memory_gates_kernel, dim3(B, H), dim3(64), 0, (hipStream_t)stream, (const float*)proj_rows, ld,
                     Gating{bias_i, bias_f, cap, i_off, f_off}, positions, cu_q, q_per_seq, state_slots, (float*)m_state, (float4*)gates, H,
                     Dv + 1, Dv + 1);
  return LAUNCH_OK();
}

extern "C" int ssd_memory_scan(const void* proj_rows, long ld, int q_off, int k_off, int v_off, float q_scale, const float* decay,
                               const void* gates, int i_off, int f_off, const float* bias_i, const float* bias_f, float cap,
                               const int64_t* positions, const int32_t* cu_q, int q_per_seq, const int32_t* state_slots, void* state,
                               void* m_state, void* out_rows, void* den_rows, int B, int H, int D, int Dv, int DP, void* stream) {
  const int mode = decay ? MODE_DECAY : (gates ? MODE_GATES : MODE_INLINE);
  if (!proj_rows || !positions || !state_slots || !state || !out_rows) return SSD_ERR_ARG;
  if (mode != MODE_DECAY && !den_rows) return SSD_ERR_ARG;
  if (mode == MODE_INLINE && (!bias_i || !bias_f || !m_state)) return SSD_ERR_ARG;
  if (B <= 0 || H <= 0 || H > 65535 || Dv <= 0 || !dp_ok(D, DP) || (!cu_q && q_per_seq <= 0) || q_off < 0 || k_off < 0 || v_off < 0 ||
      ld < (long)q_off + (long)H * D || ld < (long)k_off + (long)H * D || ld < (long)v_off + (long)H * Dv ||
      (mode == MODE_INLINE && (!(cap > 0.f) || i_off < 0 || f_off < 0 || ld < (long)i_off + H || ld < (long)f_off + H)) ||
      ((uintptr_t)state | (uintptr_t)gates) % 16)
    return SSD_ERR_SHAPE;
  const int zb = col_blocks_of(DP, mode == MODE_DECAY ? Dv : Dv + 1);
  if (zb > 65535) return SSD_ERR_SHAPE;
  const dim3 grid(B, H, zb);
  const Rows in{(const float*)proj_rows, ld, q_off, k_off, v_off, q_scale};
  const Gating gt{bias_i, bias_f, cap, i_off, f_off};
#define MEMORY(P, NJ, TB, MODE)                                                                                                        \
  hipLaunchKernelGGL((memory_scan_kernel<P, NJ, TB, MODE>), grid, dim3(256), 0, (hipStream_t)stream, in, decay, (const float4*)gates, gt, \
                     positions, cu_q, q_per_seq, state_slots, (float*)state, (float*)m_state, Dv + 1, (float*)out_rows,                  \
                     (float*)den_rows, H, D, Dv)
#define MEMORY3(P, NJ, TB)                                              \
  do {                                                                  \
    if (mode == MODE_DECAY) MEMORY(P, NJ, TB, MODE_DECAY);              \
    else if (mode == MODE_GATES) MEMORY(P, NJ, TB, MODE_GATES);         \
    else MEMORY(P, NJ, TB, MODE_INLINE);                                \
  } while (0)
  switch (DP) {
    case 32: MEMORY3(8, 1, 16); break;
    case 64: MEMORY3(16, 1, 16); break;
    case 128: MEMORY3(16, 2, 16); break;
    case 192: MEMORY3(16, 3, 16); break;
    case 256: MEMORY3(16, 4, 16); break;
    case 320: MEMORY3(16, 5, 8); break;
    case 384: MEMORY3(16, 6, 8); break;
    case 448: MEMORY3(16, 7, 8); break;
    default: MEMORY3(16, 8, 8); break;
  }
#undef MEMORY3
#undef MEMORY
  return LAUNCH_OK();
}
