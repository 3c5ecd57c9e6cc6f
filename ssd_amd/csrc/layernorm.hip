// Layer norm over an fp32 residual stream, y = (x - mean) / sqrt(var + eps) * w + b, for layers whose mixer and feed-forward are PARALLEL
// with a norm each -- x <- x + m (mixer(ln1(x)) + ff(ln2(x))) -- so that one statistic of the row serves both norms:
//  * ssd_lnorm_embed   x = table[id] as fp32 residual rows, and the first layer's one or two normed rows
//  * ssd_lnorm_tail    x += m * y (the layer's summed fp32 output row), and the next layer's one or two normed rows
//  * ssd_lnorm_rows    one normed row of x, optional row gather (the model's last norm); the bias is optional
// and for layers that normalise a sublayer's OUTPUT only -- x <- x + ln(f(x)), the sublayers read x itself:
//  * ssd_lnorm_post_tail  x += (v - mean) / sqrt(var + eps) * w with v = a fp32 row y, or pair_scale * (rms(y) * w1 + rms(y2) * w2) where a
//                      layer has two mixers side by side; and x as the next sublayer's input row in the element type
// The variance is the mean of the squared deviations (two passes over the row, which stays in registers for up to 16 entries per thread).
// One workgroup per row: 256 threads, or 1024 for rows of >= 2048 entries in batches of <= 64 rows (changes the fp32 summation ORDER only).
// `f32` selects the element type of weights and of the normed (GEMM-input) rows: 0 = bf16, 1 = fp32.
#include "common.h"

namespace {

template <typename T> __device__ __forceinline__ float ldf(const T* p);
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldf<bf16_t>(const bf16_t* p) { return bf2f(*p); }
template <typename T> __device__ __forceinline__ void stf(T* p, float v);
template <> __device__ __forceinline__ void stf<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void stf<bf16_t>(bf16_t* p, float v) { *p = (bf16_t)f2bf(v); }

template <int NT>
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  const int wave = threadIdx.x >> 6;
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[wave] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int q = 0; q < NT / 256; ++q) s += (red[4 * q] + red[4 * q + 1]) + (red[4 * q + 2] + red[4 * q + 3]);
  return s;
}

constexpr int SRC_ROW = 0, SRC_ADD = 1, SRC_EMBED = 2;

template <typename T> struct Norm { const T* w; const T* b; T* out; };

// SRC_ROW: the row x[gather[t]] as it is; SRC_ADD: x += m * y, written back; SRC_EMBED: x = table[ids[t]], written.
template <typename T, int NT, int SRC>
__global__ void __launch_bounds__(NT)
lnorm_kernel(float* __restrict__ x, const float* __restrict__ y, float m, const int64_t* __restrict__ ids, const T* __restrict__ table,
             long vocab, const int32_t* __restrict__ gather, Norm<T> n1, Norm<T> n2, float eps, int W) {
  __shared__ float red[NT / 64];
  const size_t t = blockIdx.x;
  float* xr = x + (SRC == SRC_ROW && gather ? (size_t)gather[t] : t) * W;
  const long id = SRC == SRC_EMBED ? ids[t] : 0;
  const bool ok = id >= 0 && id < vocab;
  constexpr int KEEP = 16;
  const bool kept = W <= KEEP * NT;
  auto first = [&](int c) -> float {
    float v;
    if (SRC == SRC_ADD) v = fmaf(m, y[t * W + c], xr[c]);
    else if (SRC == SRC_EMBED) v = ok ? ldf<T>(table + (size_t)id * W + c) : 0.f;
    else v = xr[c];
    if (SRC != SRC_ROW) xr[c] = v;
    return v;
  };
  float vk[KEEP], sum = 0.f;
  if (kept) {
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const int c = threadIdx.x + k * NT;
      vk[k] = c < W ? first(c) : 0.f;
      sum += vk[k];
    }
  } else {
    for (int c = threadIdx.x; c < W; c += NT) sum += first(c);
  }
  if (!n1.out) return;
  const float mean = block_sum<NT>(sum, red) / (float)W;
  float ss = 0.f;
  if (kept) {
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const float d = (int)threadIdx.x + k * NT < W ? vk[k] - mean : 0.f;
      ss = fmaf(d, d, ss);
    }
  } else {
    for (int c = threadIdx.x; c < W; c += NT) { const float d = xr[c] - mean; ss = fmaf(d, d, ss); }
  }
  const float r = 1.0f / sqrtf(block_sum<NT>(ss, red) / (float)W + eps);
  auto finish = [&](int c, float v) {
    const float z = (v - mean) * r;
    stf<T>(n1.out + t * W + c, fmaf(z, ldf<T>(n1.w + c), n1.b ? ldf<T>(n1.b + c) : 0.f));
    if (n2.out) stf<T>(n2.out + t * W + c, fmaf(z, ldf<T>(n2.w + c), ldf<T>(n2.b + c)));
  };
  if (kept) {
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const int c = threadIdx.x + k * NT;
      if (c < W) finish(c, vk[k]);
    }
  } else {
    for (int c = threadIdx.x; c < W; c += NT) finish(c, xr[c]);
  }
}

// Two sums at once through one pair of barriers.
template <int NT>
__device__ __forceinline__ float2 block_sum2(float a, float b, float2* red) {
  a = wave_sum(a);
  b = wave_sum(b);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = float2{a, b};
  __syncthreads();
  float2 s{0.f, 0.f};
#pragma unroll
  for (int q = 0; q < NT / 64; ++q) { s.x += red[q].x; s.y += red[q].y; }
  return s;
}

template <typename T> struct Sides { const float* y; const float* y2; const T* w1; const T* w2; float scale; };

// The row v stays in registers for up to 16 entries per thread; wider rows compute it again for every statistic (the same arithmetic).
template <typename T, int NT>
__global__ void __launch_bounds__(NT)
lnorm_post_tail_kernel(Sides<T> in, const T* __restrict__ w, float eps, float* __restrict__ x, T* __restrict__ next_out, int W) {
  __shared__ float red[NT / 64];
  __shared__ float2 red2[NT / 64];
  const size_t t = blockIdx.x;
  const float* y1 = in.y + t * W;
  const float* y2 = in.y2 ? in.y2 + t * W : nullptr;
  float* xr = x + t * W;
  constexpr int KEEP = 16;
  const bool kept = W <= KEEP * NT;
  float vk[KEEP], v2[KEEP];
  if (kept) {
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const int c = threadIdx.x + k * NT;
      vk[k] = c < W ? y1[c] : 0.f;
      v2[k] = c < W && y2 ? y2[c] : 0.f;
    }
  }
  float r1 = 0.f, r2 = 0.f;
  if (y2) {
    float a = 0.f, b = 0.f;
    if (kept) {
#pragma unroll
      for (int k = 0; k < KEEP; ++k) { a = fmaf(vk[k], vk[k], a); b = fmaf(v2[k], v2[k], b); }
    } else {
      for (int c = threadIdx.x; c < W; c += NT) { a = fmaf(y1[c], y1[c], a); b = fmaf(y2[c], y2[c], b); }
    }
    const float2 s = block_sum2<NT>(a, b, red2);
    r1 = 1.0f / sqrtf(s.x / (float)W + eps);
    r2 = 1.0f / sqrtf(s.y / (float)W + eps);
  }
  auto value = [&](int c, float a, float b) { return y2 ? in.scale * (a * r1 * ldf<T>(in.w1 + c) + b * r2 * ldf<T>(in.w2 + c)) : a; };
  auto again = [&](int c) { return value(c, y1[c], y2 ? y2[c] : 0.f); };
  float sum = 0.f;
  if (kept) {
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const int c = threadIdx.x + k * NT;
      if (c < W) vk[k] = value(c, vk[k], v2[k]);
      sum += vk[k];
    }
  } else {
    for (int c = threadIdx.x; c < W; c += NT) sum += again(c);
  }
  const float mean = block_sum<NT>(sum, red) / (float)W;
  float ss = 0.f;
  if (kept) {
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const float d = (int)threadIdx.x + k * NT < W ? vk[k] - mean : 0.f;
      ss = fmaf(d, d, ss);
    }
  } else {
    for (int c = threadIdx.x; c < W; c += NT) { const float d = again(c) - mean; ss = fmaf(d, d, ss); }
  }
  const float r = 1.0f / sqrtf(block_sum<NT>(ss, red) / (float)W + eps);
  auto finish = [&](int c, float v) {
    const float n = fmaf((v - mean) * r, ldf<T>(w + c), xr[c]);
    xr[c] = n;
    if (next_out) stf<T>(next_out + t * W + c, n);
  };
  if (kept) {
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const int c = threadIdx.x + k * NT;
      if (c < W) finish(c, vk[k]);
    }
  } else {
    for (int c = threadIdx.x; c < W; c += NT) finish(c, again(c));
  }
}

template <int SRC>
int launch(void* x, const void* y, float m, const int64_t* ids, const void* table, long vocab, const int32_t* gather, const void* w1,
           const void* b1, void* out1, const void* w2, const void* b2, void* out2, float eps, int T, int W, int f32, void* stream) {
  if ((out1 && (!w1 || (SRC != SRC_ROW && !b1))) || (out2 && (!out1 || !w2 || !b2))) return SSD_ERR_ARG;
  if (T <= 0 || W <= 0) return SSD_ERR_SHAPE;
#define LNORM(TY, NT)                                                                                                                  \
  hipLaunchKernelGGL((lnorm_kernel<TY, NT, SRC>), dim3(T), dim3(NT), 0, (hipStream_t)stream, (float*)x, (const float*)y, m, ids,         \
                     (const TY*)table, vocab, gather, Norm<TY>{(const TY*)w1, (const TY*)b1, (TY*)out1},                               \
                     Norm<TY>{(const TY*)w2, (const TY*)b2, (TY*)out2}, eps, W)
  if (T <= 64 && W >= 2048) {
    if (f32) LNORM(float, 1024); else LNORM(bf16_t, 1024);
  } else {
    if (f32) LNORM(float, 256); else LNORM(bf16_t, 256);
  }
#undef LNORM
  return hipGetLastError() == hipSuccess ? SSD_OK : SSD_ERR_LAUNCH;
}

}  // namespace

extern "C" int ssd_lnorm_embed(const int64_t* ids, const void* table, void* x_out, const void* w1, const void* b1, void* out1, const void* w2,
                               const void* b2, void* out2, float eps, int T, int W, long vocab, int f32, void* stream) {
  if (!ids || !table || !x_out) return SSD_ERR_ARG;
  if (vocab <= 0) return SSD_ERR_SHAPE;
  return launch<SRC_EMBED>(x_out, nullptr, 0.f, ids, table, vocab, nullptr, w1, b1, out1, w2, b2, out2, eps, T, W, f32, stream);
}

extern "C" int ssd_lnorm_tail(void* x, const void* y_rows, float mult, const void* w1, const void* b1, void* out1, const void* w2,
                              const void* b2, void* out2, float eps, int T, int W, int f32, void* stream) {
  if (!x || !y_rows) return SSD_ERR_ARG;
  return launch<SRC_ADD>(x, y_rows, mult, nullptr, nullptr, 1, nullptr, w1, b1, out1, w2, b2, out2, eps, T, W, f32, stream);
}

extern "C" int ssd_lnorm_rows(const void* x, const void* weight, const void* bias, void* out_rows, const int32_t* gather, float eps, int T,
                              int W, int f32, void* stream) {
  if (!x || !weight || !out_rows) return SSD_ERR_ARG;
  return launch<SRC_ROW>(const_cast<void*>(x), nullptr, 0.f, nullptr, nullptr, 1, gather, weight, bias, out_rows, nullptr, nullptr, nullptr,
                         eps, T, W, f32, stream);
}

extern "C" int ssd_lnorm_post_tail(void* x, const void* y_rows, const void* y2_rows, const void* w1, const void* w2, float pair_scale,
                                   const void* weight, float eps, void* next_out, int T, int W, int f32, void* stream) {
  if (!x || !y_rows || !weight || (y2_rows && (!w1 || !w2))) return SSD_ERR_ARG;
  if (T <= 0 || W <= 0) return SSD_ERR_SHAPE;
#define POST(TY, NT)                                                                                                              \
  hipLaunchKernelGGL((lnorm_post_tail_kernel<TY, NT>), dim3(T), dim3(NT), 0, (hipStream_t)stream,                                 \
                     Sides<TY>{(const float*)y_rows, (const float*)y2_rows, (const TY*)w1, (const TY*)w2, pair_scale},            \
                     (const TY*)weight, eps, (float*)x, (TY*)next_out, W)
  if (T <= 64 && W >= 2048) {
    if (f32) POST(float, 1024); else POST(bf16_t, 1024);
  } else {
    if (f32) POST(float, 256); else POST(bf16_t, 256);
  }
#undef POST
  return hipGetLastError() == hipSuccess ? SSD_OK : SSD_ERR_LAUNCH;
}
