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
// through LDS TB at a time, the next batch travels in registers meanwhile; tokens are walked in groups of U whose staged values are read one
// group ahead (a lone wave per SIMD has nothing else to hide the LDS latency behind) and whose read-outs are summed side by side; no
// barrier between tokens.  The arithmetic of a row does not depend on how a prompt is cut nor on the batch: one chain per state element in
// token order, sums in a fixed order (a group's missing tokens carry a = 1 and k = 0, which leaves the state as it is).
#include "common.h"

namespace {

constexpr int MAX_D = 512;
constexpr int MODE_GATES = 0, MODE_INLINE = 1, MODE_DECAY = 2;

struct Gating { const float* bias_i; const float* bias_f; float cap; int i_off, f_off; };

__device__ __forceinline__ float log_sigmoid_(float y) { return fminf(y, 0.f) - log1pf(expf(-fabsf(y))); }

// cap * tanh(z / cap): absolute error of a few ulp of cap, which is what an exponent's error counts in
__device__ __forceinline__ float soft_cap_(float z, float cap) {
  const float e = expf(-2.0f * fabsf(z) / cap);
  return copysignf(cap * ((1.0f - e) / (1.0f + e)), z);
}
// (a, b, exp(-m), 0) of a token from the running maxima before and after it
__device__ __forceinline__ float4 finish_gates(float2 g, float before, float m) {
  return float4{expf(g.x + before - m), expf(g.y - m), expf(-m), 0.f};
}
// The running maxima over n tokens whose log gates lie in LDS, by ONE lane: top[0] = m, the maximum before the first token, top[t + 1] = the one
// after token t (an addition and a maximum a token; the reads do not depend on the chain).  Returns the last one.
__device__ __forceinline__ float chain(const float2* pair, float* top, int n, float m) {
  constexpr int N = 16;                     // tokens whose log gates are read ahead of the chain
  top[0] = m;
  int t = 0;
  if (n >= N) {
    float2 g[N], next[N];
#pragma unroll
    for (int u = 0; u < N; ++u) g[u] = pair[u];
    for (; t + N <= n; t += N) {
      const int ahead = t + 2 * N <= n ? t + N : t;
#pragma unroll
      for (int u = 0; u < N; ++u) next[u] = pair[ahead + u];
#pragma unroll
      for (int u = 0; u < N; ++u) {
        m = fmaxf(g[u].x + m, g[u].y);
        top[t + u + 1] = m;
      }
#pragma unroll
      for (int u = 0; u < N; ++u) g[u] = next[u];
    }
  }
  for (; t < n; ++t) {
    m = fmaxf(pair[t].x + m, pair[t].y);
    top[t + 1] = m;
  }
  return m;
}

// 256 tokens a chunk: every thread prepares and finishes one token, one lane walks the chain.
__global__ void __launch_bounds__(256)
memory_gates_kernel(const float* __restrict__ proj, long ld, Gating gt, const int64_t* __restrict__ positions,
                    const int32_t* __restrict__ cu_q, int q_per_seq, const int32_t* __restrict__ state_slots, float* __restrict__ m_state,
                    float4* __restrict__ gates, int H, int copies, int ld_m) {
  constexpr int N = 256;
  __shared__ float2 pair[N];
  __shared__ float top[N + 1];              // top[t + 1] = the running maximum after token t of the chunk
  const int b = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int row0 = cu_q ? cu_q[b] : b * q_per_seq;
  const int row1 = cu_q ? cu_q[b + 1] : (b + 1) * q_per_seq;
  if (row1 <= row0) return;
  float* ms = m_state + ((size_t)state_slots[b] * H + h) * ld_m;
  float m = positions[row0] == 0 ? 0.f : ms[0];
  const float bi = gt.bias_i[h], bf = gt.bias_f[h];
  float zi = 0.f, zf = 0.f;
  auto fetch = [&](int r) {
    const int row = r + tid < row1 ? r + tid : row1 - 1;
    zi = proj[(size_t)row * ld + gt.i_off + h] + bi;
    zf = proj[(size_t)row * ld + gt.f_off + h] + bf;
  };
  fetch(row0);
  for (int r = row0; r < row1; r += N) {
    const int n = min(row1 - r, N);
    const float2 g{log_sigmoid_(soft_cap_(zf, gt.cap)), soft_cap_(zi, gt.cap)};
    pair[tid] = g;
    if (r + N < row1) fetch(r + N);
    __syncthreads();
    if (tid == 0) chain(pair, top, n, m);
    __syncthreads();
    m = top[n];
    if (tid < n) gates[(size_t)(r + tid) * H + h] = finish_gates(g, top[tid], top[tid + 1]);
    __syncthreads();
  }
  for (int c = tid; c < copies; c += N) ms[c] = m;
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
  constexpr int F = TB * DP / 256, FV = (TB * COLS + 255) / 256;       // staged q / k and v entries per thread
  constexpr int U = NJ == 1 ? 4 : (NJ == 2 ? 2 : 1);           // tokens of a group
  static_assert(TB <= 32 && TB * DP % 256 == 0 && TB % (2 * U) == 0 && U <= P, "");
  __shared__ float4 sk[TB * D4], sq[TB * D4];
  __shared__ __attribute__((aligned(16))) float2 ss[TB];              // (a, b) of the batch's tokens
  __shared__ __attribute__((aligned(16))) float sv[COLS * TB];        // [column][token]
  __shared__ float sz[2][TB], so[TB * COLS];        // exp(-m) (the batches alternate: read while the next batch is staged); read-outs
  __shared__ float2 pair[MODE == MODE_INLINE ? TB : 1];
  __shared__ float top[MODE == MODE_INLINE ? TB + 1 : 1];
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
  const float bg = MODE == MODE_INLINE ? (tid < 32 ? gt.bias_f[h] : gt.bias_i[h]) : 0.f;

  float rk[F], rq[F], rv[FV], zg = 0.f;
  float4 rg = float4{0.f, 0.f, 0.f, 0.f};
  const long step_f = 256 % DP == 0 ? (256 / DP) * in.ld : 0;   // from one staged entry of a thread to its next (DP divides 256)
  const long step_v = (256 / COLS) * in.ld;
  const float* hq = in.proj + in.q_off + (long)h * D;
  const float* hv = in.proj + in.v_off + (long)h * Dv;
  const long k_from_q = (long)in.k_off - in.q_off;
  auto fetch = [&](int r) {
    const int nb = min(row1 - r, TB);
    const float* base = hq + (size_t)(r + tid / DP) * in.ld + tid % DP;
    if (256 % DP == 0 && nb == TB && D == DP) {
#pragma unroll
      for (int f = 0; f < F; ++f) {
        rq[f] = base[f * step_f];
        rk[f] = base[f * step_f + k_from_q];
      }
    } else {
#pragma unroll
      for (int f = 0; f < F; ++f) {
        const int i = tid + 256 * f, tt = i / DP, d = i % DP;
        rq[f] = rk[f] = 0.f;
        if (tt < nb && d < D) {
          const float* src = hq + (size_t)(r + tt) * in.ld + d;
          rq[f] = *src;
          rk[f] = src[k_from_q];
        }
      }
    }
    const int c = c0 + tid % COLS;
    const float* vbase = hv + (size_t)(r + tid / COLS) * in.ld + c;
#pragma unroll
    for (int f = 0; f < FV; ++f) {
      rv[f] = c == Dv ? 1.f : 0.f;                              // (past the last column: a column of zeros that is never written)
      if (tid / COLS + f * (256 / COLS) < nb && c < Dv) rv[f] = vbase[f * step_v];
    }
    if (tid < nb) {
      if (MODE == MODE_GATES) rg = gates[(size_t)(r + tid) * H + h];
    }
    if (MODE == MODE_INLINE && tid < 64 && tid % 32 < nb) zg = in.proj[(size_t)(r + tid % 32) * in.ld + (tid < 32 ? gt.f_off : gt.i_off) + h] + bg;
  };
  auto put_out = [&](int r, int nb) {
#pragma unroll
    for (int f = 0; f < FV; ++f) {
      const int i = tid + 256 * f, tt = i / COLS, c = c0 + i % COLS;
      if (tt >= nb) continue;             // (nb <= TB: also the threads past the staged entries)
      if (c < Dv) out[((size_t)(r + tt) * H + h) * Dv + c] = so[i];
      else if (MODE != MODE_DECAY && c == Dv) den[(size_t)(r + tt) * H + h] = fmaxf(fabsf(so[i]), sz[(r - row0) / TB & 1][tt]) + 1e-6f;
    }
  };
  struct Group { float4 k[U][NJ], q[U][NJ]; float2 g[U]; float v[U]; };
  auto read = [&](Group& x, int t0) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        x.k[u][j] = sk[(t0 + u) * D4 + P * j + p];
        x.q[u][j] = sq[(t0 + u) * D4 + P * j + p];
      }
      x.g[u] = ss[t0 + u];
      x.v[u] = sv[col * TB + t0 + u];
    }
  };
  auto walk = [&](const Group& x, int t0) {
    float y[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const float a = x.g[u].x, w = MODE == MODE_DECAY ? x.v[u] : x.v[u] * x.g[u].y;
      float4 o{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        const float4 k = x.k[u][j], q = x.q[u][j];
        s[j].x = fmaf(a, s[j].x, k.x * w); s[j].y = fmaf(a, s[j].y, k.y * w);
        s[j].z = fmaf(a, s[j].z, k.z * w); s[j].w = fmaf(a, s[j].w, k.w * w);
        o.x = fmaf(s[j].x, q.x, o.x); o.y = fmaf(s[j].y, q.y, o.y);
        o.z = fmaf(s[j].z, q.z, o.z); o.w = fmaf(s[j].w, q.w, o.w);
      }
      y[u] = (o.x + o.y) + (o.z + o.w);
    }
    float mine = 0.f;                     // lane u of a column finishes token u of the group
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const float z = col_sum<P>(y[u]);
      mine = p == u ? z : mine;
    }
    if (p < U) so[(t0 + p) * COLS + col] = mine * in.q_scale;
  };
  fetch(row0);
  for (int r = row0; r < row1; r += TB) {
    const int nb = min(row1 - r, TB);
    __syncthreads();                      // the previous batch is walked: its staged rows are free, its outputs are in LDS
    if (r > row0) put_out(r - TB, TB);
#pragma unroll
    for (int f = 0; f < F; ++f) {
      reinterpret_cast<float*>(sq)[tid + 256 * f] = rq[f];
      reinterpret_cast<float*>(sk)[tid + 256 * f] = rk[f];
    }
#pragma unroll
    for (int f = 0; f < FV; ++f)
      if (tid + 256 * f < TB * COLS) sv[tid % COLS * TB + tid / COLS + f * (256 / COLS)] = rv[f];
    if (MODE == MODE_INLINE && tid < 64) {
      // lanes t and t + 32 prepare token t's forget and input gate
      const float c = soft_cap_(zg, gt.cap), lf = log_sigmoid_(c);
      if (tid % 32 < TB) (tid < 32 ? pair[tid % 32].x : pair[tid % 32].y) = tid < 32 ? lf : c;
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_s_waitcnt(0xc07f);               // lgkmcnt(0): this wave's LDS writes have landed
      if (tid == 0) m = chain(pair, top, nb, m);
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_s_waitcnt(0xc07f);
      if (tid < nb) rg = finish_gates(pair[tid], top[tid], top[tid + 1]);
    }
    if (MODE == MODE_DECAY) rg.x = fixed;
    if (tid < TB) {
      ss[tid] = tid < nb ? float2{rg.x, rg.y} : float2{1.f, 0.f};
      sz[(r - row0) / TB & 1][tid] = rg.z;
    }
    __syncthreads();
    if (r + TB < row1) fetch(r + TB);
    Group x0, x1;
    read(x0, 0);
    if (nb == TB) {
#pragma unroll 1
      for (int t = 0; t < TB; t += 2 * U) {
        read(x1, t + U);
        walk(x0, t);
        read(x0, min(t + 2 * U, TB - U));
        walk(x1, t + U);
      }
    } else {
      for (int t = 0; t < nb; t += U) {
        if (t > 0) read(x0, t);
        walk(x0, t);
      }
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
  hipLaunchKernelGGL(memory_gates_kernel, dim3(B, H), dim3(256), 0, (hipStream_t)stream, (const float*)proj_rows, ld,
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
  if (!cu_q && q_per_seq <= 8 && DP <= 256) {          // decoding: a batch is staged for few tokens
    switch (DP) {
      case 32: MEMORY3(8, 1, 8); break;
      case 64: MEMORY3(16, 1, 8); break;
      case 128: MEMORY3(16, 2, 8); break;
      case 192: MEMORY3(16, 3, 8); break;
      default: MEMORY3(16, 4, 8); break;
    }
    return LAUNCH_OK();
  }
  switch (DP) {
    case 32: MEMORY3(8, 1, 32); break;
    case 64: MEMORY3(16, 1, 32); break;
    case 128: MEMORY3(16, 2, 32); break;
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
