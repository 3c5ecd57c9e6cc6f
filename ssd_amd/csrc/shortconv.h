// Short causal convolutions over time on columns of fp32 projection rows, shared by the mixers that have one:
//     y_t[c] = sum_j w[c][j] * u_(t - (taps - 1) + j)[c],   u = 0 before the sequence's first token
// The inputs of the taps - 1 tokens before a portion come from the sequence's slot: conv_state[slots][taps - 1][C] fp32, saved row i = the
// input of position p0 - (taps - 1) + i when the portion starts at position p0.  The kernels that convolve READ the slot; a later launch
// of the same forward (the mixer's scan) writes it back with save_conv_state, so no workgroup reads what another one overwrites.
#pragma once
#include "common.h"

constexpr int CONV_MAX_TAPS = 16;

// Sequence of token row t in a varlen batch (cu_q) or a batch of q_per_seq rows per sequence.
__device__ __forceinline__ int seq_of_row(const int32_t* cu_q, int q_per_seq, int B, int t) {
  if (!cu_q) return t / q_per_seq;
  int lo = 0, hi = B;
  while (hi - lo > 1) { const int mid = (lo + hi) >> 1; if (cu_q[mid] <= t) lo = mid; else hi = mid; }
  return lo;
}

// Channel c of the convolution at row t of a portion that starts at row row0 / position p0, on top of `acc`.  col: the channel's column
// in the projection rows; w: its weights; st: the slot's saved rows (row stride C).  TAPS: the tap count, or 0 for any (`taps`).  All
// inputs are loaded before the first product (a load that must not count reads the current row's entry and is replaced by zero), so the
// taps cost one memory round trip.
template <typename T, int TAPS>
__device__ __forceinline__ float conv_at(const float* __restrict__ proj, long ld, long col, int c, int C, const T* __restrict__ w, int taps,
                                         const float* __restrict__ st, int t, int row0, long p0, float acc) {
  constexpr int N = TAPS > 0 ? TAPS : CONV_MAX_TAPS;
  const int n = TAPS > 0 ? TAPS : taps;
  const float* cur = proj + (size_t)t * ld + col;
  float v[N], wv[N];
#pragma unroll
  for (int j = 0; j < N; ++j) {
    v[j] = wv[j] = 0.f;
    if (TAPS == 0 && j >= n) continue;
    const int back = n - 1 - j, k = row0 - (t - back);     // k > 0: so many tokens before the portion's first row
    const bool saved = k > 0, zero = saved && p0 - k < 0;
    const float* src = zero ? cur : (saved ? st + (size_t)(n - 1 - k) * C + c : cur - (size_t)back * ld);
    v[j] = *src;
    if (zero) v[j] = 0.f;
    if constexpr (sizeof(T) == 2) wv[j] = bf2f(w[j]); else wv[j] = w[j];
  }
#pragma unroll
  for (int j = 0; j < N; ++j)
    if (TAPS > 0 || j < n) acc = fmaf(wv[j], v[j], acc);
  return acc;
}
// runs BODY(TAPS) with the tap count as a constant for the usual counts
#define CONV_TAPS(taps, BODY)      \
  do {                             \
    switch (taps) {                \
      case 2: BODY(2); break;      \
      case 3: BODY(3); break;      \
      case 4: BODY(4); break;      \
      default: BODY(0); break;     \
    }                              \
  } while (0)

// Channels [c_begin, c_end) of the slot's saved convolution inputs: saved row i holds the input of position p0 + n - (taps - 1) + i.
__device__ __forceinline__ void save_conv_state(const float* proj, long ld, int conv_off, int C, float* conv_state, int taps, int slot,
                                                int row0, int row1, long p0, int c_begin, int c_end) {
  const int n = row1 - row0, K1 = taps - 1;
  float* st = conv_state + (size_t)slot * K1 * C;
  for (int c = c_begin + threadIdx.x; c < c_end; c += 256) {
    float keep[CONV_MAX_TAPS];
#pragma unroll
    for (int i = 0; i < CONV_MAX_TAPS; ++i) {
      keep[i] = 0.f;
      if (i < K1) {
        const long rel = (long)n - K1 + i;                // position relative to the portion's first row
        if (rel >= 0) keep[i] = proj[(size_t)(row0 + rel) * ld + conv_off + c];
        else if (p0 + rel >= 0) keep[i] = st[(size_t)(i + n) * C + c];
      }
    }
#pragma unroll
    for (int i = 0; i < CONV_MAX_TAPS; ++i)
      if (i < K1) st[(size_t)i * C + c] = keep[i];
  }
}
