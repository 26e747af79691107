// Norms of a layer arrangement that norms a sublayer's output before it joins the residual
// stream ("sandwich": x += N_b(f(N_a(x)))), and the gated norm behind a recurrent mixer.
// All sums, inverse roots and the residual stream are float.
#include "common.h"

// ---------------------------------------------------------------- post-norm + residual add + next pre-norm
// Row r = rows ? rows[i] : i.
//   v   = (y ? y[r] : 0) + parts[0][r] + parts[1][r] + ... (+ bias)   (the sublayer's output; parts added in order)
//   x   = h[r] + v * rsqrt(mean(v^2) + eps) * wb                 (float)
//         or, where wb is null (a sublayer's output that joins the stream under a constant only), h[r] + v * plain_scale
//   if (!rows) h[r] = x
//   if (out)   out[i] = T( x * rsqrt(mean(x^2) + eps_out) * w ),   or T(x) where w is null
// One block per output row; the row is kept in LDS between the passes (hidden floats).
template <typename T>
__global__ void __launch_bounds__(256)
postnorm_add_rmsnorm_kernel(float* __restrict__ h, const T* __restrict__ y, const float* __restrict__ parts,
                            int n_parts, long long part_stride, const float* __restrict__ bias,
                            const float* __restrict__ wb,
                            const float* __restrict__ w, T* __restrict__ out, const int* __restrict__ rows,
                            int hidden, float eps, float eps_out, float plain_scale) {
  extern __shared__ float row[];
  __shared__ float red[32];
  const long long i = blockIdx.x;
  const long long r = rows ? (long long)rows[i] : i;
  float* hr = h + r * hidden;
  float ss = 0.f;
  for (int c = threadIdx.x; c < hidden; c += blockDim.x) {
    float v = y ? to_f32(y[r * hidden + c]) : 0.f;
    for (int p = 0; p < n_parts; ++p) v += parts[p * part_stride + r * hidden + c];
    if (bias) v += bias[c];
    row[c] = v;
    ss += v * v;
  }
  ss = block_sum(ss, red);
  const float inv_b = wb ? rsqrtf(ss / (float)hidden + eps) : plain_scale;
  float ss2 = 0.f;
  for (int c = threadIdx.x; c < hidden; c += blockDim.x) {
    const float x = hr[c] + row[c] * inv_b * (wb ? wb[c] : 1.f);
    if (!rows) hr[c] = x;
    row[c] = x;
    ss2 += x * x;
  }
  if (!out) return;
  T* o = out + i * hidden;
  if (!w) {          // the reader takes the stream itself: no norm, the row in the activation type
    for (int c = threadIdx.x; c < hidden; c += blockDim.x) o[c] = from_f32<T>(row[c]);
    return;
  }
  ss2 = block_sum(ss2, red);
  const float inv = rsqrtf(ss2 / (float)hidden + eps_out);
  for (int c = threadIdx.x; c < hidden; c += blockDim.x) o[c] = from_f32<T>(row[c] * inv * w[c]);
}

// ---------------------------------------------------------------- norm of float rows times a sigmoid gate
//   out[t, c] = T( o[t, c] * rsqrt(mean_c(o[t]^2) + eps) * w[c] * sigmoid(g[t * g_stride + c]) )
// o is float (the output of a recurrence), g lives in a wider row of the activation type.
template <typename T>
__global__ void __launch_bounds__(256)
gated_rmsnorm_kernel(T* __restrict__ out, const float* __restrict__ o, const T* __restrict__ g,
                     long long g_stride, const float* __restrict__ w, int width, float eps) {
  __shared__ float red[32];
  const long long t = blockIdx.x;
  const float* x = o + t * width;
  float ss = 0.f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) ss += x[c] * x[c];
  ss = block_sum(ss, red);
  const float inv = rsqrtf(ss / (float)width + eps);
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const float gate = 1.f / (1.f + expf(-to_f32(g[t * g_stride + c])));
    out[t * width + c] = from_f32<T>(x[c] * inv * w[c] * gate);
  }
}

// The same for widths that are multiples of 4: 16 bytes of the float arrays a lane, every load of a pass asked
// for before the sums (a decode step has few rows: what a row costs is its chain of dependent loads).
template <typename T> struct SnVec4;
template <> struct SnVec4<float> { typedef float4 type; };
template <> struct SnVec4<bf16_t> { typedef __attribute__((ext_vector_type(4))) __bf16 type; };
template <typename T> __device__ __forceinline__ float4 sn_load4(const T* p) {
  const typename SnVec4<T>::type v = *(const typename SnVec4<T>::type*)p;
  return float4{to_f32<T>(v[0]), to_f32<T>(v[1]), to_f32<T>(v[2]), to_f32<T>(v[3])};
}
template <> __device__ __forceinline__ float4 sn_load4<float>(const float* p) { return *(const float4*)p; }
template <typename T> __device__ __forceinline__ void sn_store4(T* p, float4 v) {
  typename SnVec4<T>::type o;
  o[0] = from_f32<T>(v.x); o[1] = from_f32<T>(v.y); o[2] = from_f32<T>(v.z); o[3] = from_f32<T>(v.w);
  *(typename SnVec4<T>::type*)p = o;
}
template <> __device__ __forceinline__ void sn_store4<float>(float* p, float4 v) { *(float4*)p = v; }

// A causal filter over time behind the next norm, for steps with one token a request (row i is request i): with
// x the normed row, out = x + sum_j wt[lags - j] * (the input j tokens back), the last `lags` inputs read from and left
// in the request's state row [lags][hidden] (token_filter.hip has the form for any step).
struct SnFilter {
  const float* wt;         // [lags + 1][hidden]
  float* state;            // [slots + 1][lags][hidden]
  const int* slot_ids;
  int lags;
};

#define SN_V 4          // 16-byte pieces a thread of a block of 256: rows of up to 4 * SN_V * 256 = 4,096 floats
#define SN_FEW_ROWS 64  // up to so many rows a row gets a thread for each of its 16-byte pieces
#define SN_PARTS 4      // partial results a thread with one piece asks for at once

// V pieces a thread, blocks of `blockDim.x` threads; L > 0: with a filter of up to L lags (L = 0: none).  Everything a
// row needs is asked for before its first sum (the filter's inputs and weights too): a row's time is its chain of loads.
template <typename T, int V, int L>
__global__ void __launch_bounds__(V == 1 ? 1024 : 256)
postnorm_add_rmsnorm_vec_kernel(float* __restrict__ h, const T* __restrict__ y, const float* __restrict__ parts,
                                int n_parts, long long part_stride, const float* __restrict__ bias,
                                const float* __restrict__ wb,
                                const float* __restrict__ w, T* __restrict__ out, const int* __restrict__ rows,
                                int hidden, float eps, float eps_out, float plain_scale, SnFilter f) {
  __shared__ float red[32];
  const long long i = blockIdx.x;
  const long long r = rows ? (long long)rows[i] : i;
  const int step = blockDim.x * 4;
  const float4 zero4 = float4{0.f, 0.f, 0.f, 0.f};
  float4 v[V], x[V], b[V], g[V];
  float4 past[L ? L * V : 1], tap[L ? (L + 1) * V : 1];
  float* st = nullptr;
  if constexpr (L > 0) st = f.state + (long long)f.slot_ids[r] * f.lags * hidden;
  float ss = 0.f;
#pragma unroll
  for (int q = 0; q < V; ++q) {
    const int c = threadIdx.x * 4 + q * step;
    const int cc = c < hidden ? c : 0;           // a piece beyond the row reads the row's first piece, its share is left out
    v[q] = y ? sn_load4<T>(y + r * hidden + cc) : zero4;
    x[q] = *(const float4*)(h + r * hidden + cc);
    b[q] = wb ? *(const float4*)(wb + cc) : float4{1.f, 1.f, 1.f, 1.f};
    g[q] = w ? *(const float4*)(w + cc) : zero4;
    if constexpr (L > 0) {
#pragma unroll
      for (int j = 0; j < L; ++j)
        past[q * L + j] = j < f.lags ? *(const float4*)(st + (long long)j * hidden + cc) : zero4;
#pragma unroll
      for (int j = 0; j <= L; ++j)
        tap[q * (L + 1) + j] = j <= f.lags ? *(const float4*)(f.wt + (long long)j * hidden + cc) : zero4;
    }
  }
  constexpr int PB = V == 1 ? SN_PARTS : 1;
  for (int p0 = 0; p0 < n_parts; p0 += PB) {
    float4 t[PB][V];
#pragma unroll
    for (int p = 0; p < PB; ++p)
#pragma unroll
      for (int q = 0; q < V; ++q) {
        const int c = threadIdx.x * 4 + q * step;
        t[p][q] = p0 + p < n_parts ? *(const float4*)(parts + (p0 + p) * part_stride + r * hidden + (c < hidden ? c : 0)) : zero4;
      }
#pragma unroll
    for (int p = 0; p < PB; ++p)
#pragma unroll
      for (int q = 0; q < V; ++q) { v[q].x += t[p][q].x; v[q].y += t[p][q].y; v[q].z += t[p][q].z; v[q].w += t[p][q].w; }
  }
  if (bias) {
#pragma unroll
    for (int q = 0; q < V; ++q) {
      const int c = threadIdx.x * 4 + q * step;
      const float4 t = *(const float4*)(bias + (c < hidden ? c : 0));
      v[q].x += t.x; v[q].y += t.y; v[q].z += t.z; v[q].w += t.w;
    }
  }
#pragma unroll
  for (int q = 0; q < V; ++q)
    if (threadIdx.x * 4 + q * step < hidden) ss += v[q].x * v[q].x + v[q].y * v[q].y + v[q].z * v[q].z + v[q].w * v[q].w;
  float inv_b = plain_scale;
  if (wb) {
    ss = block_sum(ss, red);
    inv_b = rsqrtf(ss / (float)hidden + eps);
  }
  float ss2 = 0.f;
#pragma unroll
  for (int q = 0; q < V; ++q) {
    const int c = threadIdx.x * 4 + q * step;
    x[q].x += v[q].x * inv_b * b[q].x; x[q].y += v[q].y * inv_b * b[q].y;
    x[q].z += v[q].z * inv_b * b[q].z; x[q].w += v[q].w * inv_b * b[q].w;
    if (c < hidden) {
      if (!rows) *(float4*)(h + r * hidden + c) = x[q];
      ss2 += x[q].x * x[q].x + x[q].y * x[q].y + x[q].z * x[q].z + x[q].w * x[q].w;
    }
  }
  if (!out) return;
  if (!w) {          // the reader takes the stream itself: no norm, the row in the activation type
#pragma unroll
    for (int q = 0; q < V; ++q) {
      const int c = threadIdx.x * 4 + q * step;
      if (c < hidden) sn_store4<T>(out + i * hidden + c, x[q]);
    }
    return;
  }
  ss2 = block_sum(ss2, red);
  const float inv = rsqrtf(ss2 / (float)hidden + eps_out);
#pragma unroll
  for (int q = 0; q < V; ++q) {
    const int c = threadIdx.x * 4 + q * step;
    if (c >= hidden) continue;
    const float4 o = float4{x[q].x * inv * g[q].x, x[q].y * inv * g[q].y, x[q].z * inv * g[q].z, x[q].w * inv * g[q].w};
    if constexpr (L > 0) {
      // the input in the activation type, as a later step reads it
      const float4 u = float4{to_f32(from_f32<T>(o.x)), to_f32(from_f32<T>(o.y)), to_f32(from_f32<T>(o.z)), to_f32(from_f32<T>(o.w))};
      float4 acc = zero4;
#pragma unroll
      for (int j = 0; j <= L; ++j) {
        if (j > f.lags) break;
        const float4 in = j < f.lags ? past[q * L + (j < L ? j : 0)] : u;
        const float4 k = tap[q * (L + 1) + j];
        acc = float4{fmaf(k.x, in.x, acc.x), fmaf(k.y, in.y, acc.y), fmaf(k.z, in.z, acc.z), fmaf(k.w, in.w, acc.w)};
        if (j > 0) *(float4*)(st + (long long)(j - 1) * hidden + c) = in;
      }
      sn_store4<T>(out + i * hidden + c, float4{acc.x + u.x, acc.y + u.y, acc.z + u.z, acc.w + u.w});
    } else {
      sn_store4<T>(out + i * hidden + c, o);
    }
  }
}

#define DEFINE_SANDWICH(SUF, T)                                                                          \
  extern "C" int jv_postnorm_add_rmsnorm_##SUF(float* h, const void* y, const float* parts, int n_parts, \
                                               long long part_stride, const float* bias,               \
                                               const float* wb, const float* w,                         \
                                               void* out, const int* rows, int n_out, int hidden,        \
                                               float eps, float eps_out, float plain_scale,              \
                                               void* stream) {                                           \
    if (n_out <= 0 || hidden <= 0) return 0;                                                             \
    if ((!y && n_parts <= 0) || hidden > 16384) return (int)hipErrorInvalidValue;                        \
    if (hidden % 4 == 0 && hidden <= 4 * SN_V * 256) {                                                   \
      const bool few = n_out <= SN_FEW_ROWS;                                                             \
      auto kernel = few || hidden <= 1024 ? postnorm_add_rmsnorm_vec_kernel<T, 1, 0>                     \
                    : hidden <= 2048 ? postnorm_add_rmsnorm_vec_kernel<T, 2, 0> : postnorm_add_rmsnorm_vec_kernel<T, SN_V, 0>; \
      hipLaunchKernelGGL(kernel, dim3(n_out), dim3(few ? (hidden / 4 + 63) / 64 * 64 : 256), 0,          \
                         (hipStream_t)stream, h, (const T*)y, parts, n_parts, part_stride, bias, wb, w,  \
                         (T*)out, rows, hidden, eps, eps_out, plain_scale, SnFilter{});                  \
      return JV_LAUNCH_CHECK();                                                                          \
    }                                                                                                    \
    hipLaunchKernelGGL(postnorm_add_rmsnorm_kernel<T>, dim3(n_out), dim3(256), hidden * sizeof(float),   \
                       (hipStream_t)stream, h, (const T*)y, parts, n_parts, part_stride, bias, wb, w,    \
                       (T*)out,                                                                          \
                       rows, hidden, eps, eps_out, plain_scale);                                         \
    return JV_LAUNCH_CHECK();                                                                            \
  }                                                                                                      \
  extern "C" int jv_norm_filter_##SUF(float* h, const void* y, const float* parts, int n_parts,           \
                                      long long part_stride, const float* wb, const float* w, void* out,  \
                                      int n, int hidden, float eps, float eps_out, const float* wt,        \
                                      float* state, const int* slot_ids, int taps, void* stream) {         \
    if (n <= 0 || hidden <= 0) return 0;                                                                 \
    if (hidden % 4 || hidden > 4 * SN_V * 256 || !w || !out || !wt || taps < 1 || taps > 8 ||            \
        (taps > 1 && (!state || !slot_ids)))                                                             \
      return (int)hipErrorInvalidValue;                                                                  \
    auto kernel = taps <= 4 ? postnorm_add_rmsnorm_vec_kernel<T, 1, 3> : postnorm_add_rmsnorm_vec_kernel<T, 1, 7>; \
    hipLaunchKernelGGL(kernel, dim3(n), dim3((hidden / 4 + 63) / 64 * 64), 0,                            \
                       (hipStream_t)stream, h, (const T*)y, parts, n_parts, part_stride,                 \
                       (const float*)nullptr, wb, w, (T*)out, (const int*)nullptr, hidden, eps, eps_out,  \
                       1.f, SnFilter{wt, state, slot_ids, taps - 1});                                    \
    return JV_LAUNCH_CHECK();                                                                            \
  }                                                                                                      \
  extern "C" int jv_gated_rmsnorm_##SUF(void* out, const float* o, const void* g, long long g_stride,    \
                                        const float* w, int n, int width, float eps, void* stream) {     \
    if (n <= 0 || width <= 0) return 0;                                                                  \
    hipLaunchKernelGGL(gated_rmsnorm_kernel<T>, dim3(n), dim3(256), 0, (hipStream_t)stream, (T*)out, o,  \
                       (const T*)g, g_stride, w, width, eps);                                            \
    return JV_LAUNCH_CHECK();                                                                            \
  }

DEFINE_SANDWICH(bf16, bf16_t)
DEFINE_SANDWICH(f32, float)
