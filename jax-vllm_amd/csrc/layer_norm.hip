// Layer norm (mean taken off, weight and bias) of the float residual stream, fused with the residual step before it:
// what a sublayer handed on joins the stream as it is, under a constant, under an RMS norm of its own, or as the sum of
// two outputs that each have an RMS norm of their own (two mixers side by side).
//
// Row r = rows ? rows[i] : i.
//   v_s = (y_s ? y_s[r] : 0) + parts_s[0][r] + parts_s[1][r] + ...           (s = 0, or 0 and 1; parts added in order)
//   x   = h[r] + sum_s ( w_s ? v_s * rsqrt(mean(v_s^2) + eps_s) * w_s : v_s * scale_s )          (float)
//   if (!rows) h[r] = x
//   out[i] = T( (x - mean(x)) * rsqrt(mean((x - mean(x))^2) + eps) * w + bias )
// The mean of x is the mean of its summands, so one exchange over the block gives the mean squares of v_s and the mean
// of x, a second one the variance.
#include "common.h"

template <typename T> struct LnShare {
  const T* y;              // rows of the activation type, or null
  const float* parts;      // float stack [n][rows][hidden], or null
  int n;
  long long stride;
  const float* w;          // weight of the output's own norm, or null
  float eps, scale;
};

// Sums of N values a thread over a whole block of up to 1024 threads; `red` is shared scratch of >= 16 N floats.
template <int N>
__device__ __forceinline__ void ln_block_sums(float (&v)[N], float* red) {
  const int lane = threadIdx.x & (JV_WAVE - 1), wid = threadIdx.x / JV_WAVE;
  const int nw = (blockDim.x + JV_WAVE - 1) / JV_WAVE;
#pragma unroll
  for (int i = 0; i < N; ++i) v[i] = wave_sum(v[i]);
  __syncthreads();         // protects `red` against a previous use
  if (lane == 0) {
#pragma unroll
    for (int i = 0; i < N; ++i) red[i * 16 + wid] = v[i];
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < N; ++i) {
    float t = lane < nw ? red[i * 16 + lane] : 0.f;
#pragma unroll
    for (int o = 8; o > 0; o >>= 1) t += __shfl_xor(t, o, JV_WAVE);     // at most 16 waves: the other lanes hold zeros
    v[i] = __shfl(t, 0, JV_WAVE);
  }
}

template <typename T> struct LnVec4;
template <> struct LnVec4<float> { typedef float type __attribute__((ext_vector_type(4))); };
template <> struct LnVec4<bf16_t> { typedef bf16_t type __attribute__((ext_vector_type(4))); };
template <typename T> __device__ __forceinline__ void ln_load4(const T* p, float (&v)[4]) {
  const typename LnVec4<T>::type x = *(const typename LnVec4<T>::type*)p;
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] = to_f32<T>(x[e]);
}
template <typename T> __device__ __forceinline__ void ln_store4(T* p, const float (&v)[4]) {
  typename LnVec4<T>::type x;
#pragma unroll
  for (int e = 0; e < 4; ++e) x[e] = from_f32<T>(v[e]);
  *(typename LnVec4<T>::type*)p = x;
}

#define LN_MAX_V 4      // 16-byte pieces a thread of a block of 256: rows of up to 4,096 floats
#define LN_FEW_ROWS 64  // up to so many rows a row gets a thread for each of its 16-byte pieces
#define LN_PARTS 4      // partial results a thread with one piece asks for at once

// SHARES: how many outputs join (0, 1, 2).  Every load of a pass is asked for before its first sum.
template <typename T, int V, int SHARES>
__global__ void __launch_bounds__(V == 1 ? 1024 : 256)
add_layernorm_vec_kernel(float* __restrict__ h, LnShare<T> sa, LnShare<T> sb, const float* __restrict__ w,
                         const float* __restrict__ bias, T* __restrict__ out, const int* __restrict__ rows, int hidden,
                         float eps) {
  __shared__ float red[16 * 5];
  const long long i = blockIdx.x;
  const long long r = rows ? (long long)rows[i] : i;
  const int step = blockDim.x * 4;
  constexpr int NS = SHARES ? SHARES : 1;
  float x[V][4], v[NS][V][4], wn[NS][V][4], g[V][4], b[V][4];
#pragma unroll
  for (int q = 0; q < V; ++q) {
    const int c = threadIdx.x * 4 + q * step;
    const int cc = c < hidden ? c : 0;           // a piece beyond the row reads the row's first piece, its share is left out
    ln_load4<float>(h + r * hidden + cc, x[q]);
    ln_load4<float>(w + cc, g[q]);
    ln_load4<float>(bias + cc, b[q]);
#pragma unroll
    for (int s = 0; s < SHARES; ++s) {
      const LnShare<T>& S = s ? sb : sa;
#pragma unroll
      for (int e = 0; e < 4; ++e) { v[s][q][e] = 0.f; wn[s][q][e] = 1.f; }
      if (S.y) ln_load4<T>(S.y + r * hidden + cc, v[s][q]);
      if (S.w) ln_load4<float>(S.w + cc, wn[s][q]);
    }
  }
  constexpr int PB = V == 1 ? LN_PARTS : 1;
#pragma unroll
  for (int s = 0; s < SHARES; ++s) {
    const LnShare<T>& S = s ? sb : sa;
    for (int p0 = 0; p0 < S.n; p0 += PB) {
      float t[PB][V][4];
#pragma unroll
      for (int p = 0; p < PB; ++p)
#pragma unroll
        for (int q = 0; q < V; ++q) {
          const int c = threadIdx.x * 4 + q * step;
          const int pp = p0 + p < S.n ? p0 + p : S.n - 1;      // a repeat is left out of the sum
          ln_load4<float>(S.parts + pp * S.stride + r * hidden + (c < hidden ? c : 0), t[p][q]);
        }
#pragma unroll
      for (int p = 0; p < PB; ++p)
#pragma unroll
        for (int q = 0; q < V; ++q)
#pragma unroll
          for (int e = 0; e < 4; ++e) v[s][q][e] += p0 + p < S.n ? t[p][q][e] : 0.f;
    }
  }
  // sum of h, and per share the sum of squares and the sum under its weight
  float sums[1 + 2 * SHARES];
#pragma unroll
  for (int k = 0; k < 1 + 2 * SHARES; ++k) sums[k] = 0.f;
#pragma unroll
  for (int q = 0; q < V; ++q) {
    if (threadIdx.x * 4 + q * step >= hidden) continue;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      sums[0] += x[q][e];
#pragma unroll
      for (int s = 0; s < SHARES; ++s) {
        sums[1 + 2 * s] = fmaf(v[s][q][e], v[s][q][e], sums[1 + 2 * s]);
        sums[2 + 2 * s] = fmaf(v[s][q][e], wn[s][q][e], sums[2 + 2 * s]);
      }
    }
  }
  ln_block_sums(sums, red);
  const float inv_n = 1.f / (float)hidden;
  float mean = sums[0];
  float inv[NS];
#pragma unroll
  for (int s = 0; s < SHARES; ++s) {
    const LnShare<T>& S = s ? sb : sa;
    inv[s] = S.w ? rsqrtf(sums[1 + 2 * s] * inv_n + S.eps) : S.scale;
    mean = fmaf(inv[s], sums[2 + 2 * s], mean);
  }
  mean *= inv_n;
  float var[1] = {0.f};
#pragma unroll
  for (int q = 0; q < V; ++q) {
    const int c = threadIdx.x * 4 + q * step;
#pragma unroll
    for (int e = 0; e < 4; ++e)
#pragma unroll
      for (int s = 0; s < SHARES; ++s) x[q][e] += v[s][q][e] * inv[s] * wn[s][q][e];
    if (c < hidden) {
      if (SHARES && !rows) ln_store4<float>(h + r * hidden + c, x[q]);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float d = x[q][e] - mean;
        var[0] = fmaf(d, d, var[0]);
      }
    }
  }
  ln_block_sums(var, red);
  const float scale = rsqrtf(var[0] * inv_n + eps);
#pragma unroll
  for (int q = 0; q < V; ++q) {
    const int c = threadIdx.x * 4 + q * step;
    if (c >= hidden) continue;
    float o[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = fmaf((x[q][e] - mean) * scale, g[q][e], b[q][e]);
    ln_store4<T>(out + i * hidden + c, o);
  }
}

// Any width up to 16,384: the row of x in LDS between the passes, the outputs read twice.
template <typename T>
__device__ __forceinline__ float ln_share_at(const LnShare<T>& S, long long at) {
  float v = S.y ? to_f32(S.y[at]) : 0.f;
  for (int p = 0; p < S.n; ++p) v += S.parts[p * S.stride + at];
  return v;
}
template <typename T>
__global__ void __launch_bounds__(256)
add_layernorm_kernel(float* __restrict__ h, LnShare<T> sa, LnShare<T> sb, int shares, const float* __restrict__ w,
                     const float* __restrict__ bias, T* __restrict__ out, const int* __restrict__ rows, int hidden,
                     float eps) {
  extern __shared__ float row[];
  __shared__ float red[16 * 5];
  const long long i = blockIdx.x;
  const long long r = rows ? (long long)rows[i] : i;
  float sq[2] = {0.f, 0.f};
  for (int c = threadIdx.x; c < hidden; c += blockDim.x) {
    if (shares > 0 && sa.w) { const float v = ln_share_at(sa, r * hidden + c); sq[0] = fmaf(v, v, sq[0]); }
    if (shares > 1 && sb.w) { const float v = ln_share_at(sb, r * hidden + c); sq[1] = fmaf(v, v, sq[1]); }
  }
  ln_block_sums(sq, red);
  const float ia = sa.w ? rsqrtf(sq[0] / (float)hidden + sa.eps) : sa.scale;
  const float ib = sb.w ? rsqrtf(sq[1] / (float)hidden + sb.eps) : sb.scale;
  float sum[1] = {0.f};
  for (int c = threadIdx.x; c < hidden; c += blockDim.x) {
    float x = h[r * hidden + c];
    if (shares > 0) x += ln_share_at(sa, r * hidden + c) * ia * (sa.w ? sa.w[c] : 1.f);
    if (shares > 1) x += ln_share_at(sb, r * hidden + c) * ib * (sb.w ? sb.w[c] : 1.f);
    if (shares && !rows) h[r * hidden + c] = x;
    row[c] = x;
    sum[0] += x;
  }
  ln_block_sums(sum, red);
  const float mean = sum[0] / (float)hidden;
  float var[1] = {0.f};
  for (int c = threadIdx.x; c < hidden; c += blockDim.x) var[0] = fmaf(row[c] - mean, row[c] - mean, var[0]);
  ln_block_sums(var, red);
  const float scale = rsqrtf(var[0] / (float)hidden + eps);
  for (int c = threadIdx.x; c < hidden; c += blockDim.x) out[i * hidden + c] = from_f32<T>(fmaf((row[c] - mean) * scale, w[c], bias[c]));
}

template <typename T, int V>
static void launch_add_layernorm(int shares, int n_out, int threads, hipStream_t s, float* h, const LnShare<T>& a,
                                 const LnShare<T>& b, const float* w, const float* bias, T* out, const int* rows,
                                 int hidden, float eps) {
  auto kernel = shares == 0 ? add_layernorm_vec_kernel<T, V, 0> : shares == 1 ? add_layernorm_vec_kernel<T, V, 1>
                                                                             : add_layernorm_vec_kernel<T, V, 2>;
  hipLaunchKernelGGL(kernel, dim3(n_out), dim3(threads), 0, s, h, a, b, w, bias, out, rows, hidden, eps);
}

template <typename T>
static int add_layernorm_entry(float* h, int shares, const LnShare<T>& a, const LnShare<T>& b, const float* w,
                               const float* bias, T* out, const int* rows, int n_out, int hidden, float eps, int vec,
                               void* stream) {
  if (n_out <= 0 || hidden <= 0) return 0;
  if (!h || !w || !bias || !out || hidden > 16384 || shares < 0 || shares > 2) return (int)hipErrorInvalidValue;
  if (shares > 0 && ((!a.y && a.n <= 0) || (a.n > 0 && !a.parts))) return (int)hipErrorInvalidValue;
  if (shares > 1 && ((!b.y && b.n <= 0) || (b.n > 0 && !b.parts))) return (int)hipErrorInvalidValue;
  hipStream_t s = (hipStream_t)stream;
  if (vec && hidden % 4 == 0 && hidden <= 4 * LN_MAX_V * 256) {
    if (n_out <= LN_FEW_ROWS || hidden <= 1024)
      launch_add_layernorm<T, 1>(shares, n_out, (hidden / 4 + 63) / 64 * 64, s, h, a, b, w, bias, out, rows, hidden, eps);
    else if (hidden <= 2048)
      launch_add_layernorm<T, 2>(shares, n_out, 256, s, h, a, b, w, bias, out, rows, hidden, eps);
    else
      launch_add_layernorm<T, LN_MAX_V>(shares, n_out, 256, s, h, a, b, w, bias, out, rows, hidden, eps);
    return JV_LAUNCH_CHECK();
  }
  hipLaunchKernelGGL(add_layernorm_kernel<T>, dim3(n_out), dim3(256), (size_t)hidden * sizeof(float), s, h, a, b, shares, w,
                     bias, out, rows, hidden, eps);
  return JV_LAUNCH_CHECK();
}

// shares 0..2 of the outputs (ya, pa, ...), (yb, pb, ...) join the stream; `vec`: every pointer and stride allows 16-byte
// pieces of the float arrays (and 8 bytes of bfloat16).
#define DEFINE_LAYER_NORM(SUF, T)                                                                                 \
  extern "C" int jv_add_layernorm_##SUF(float* h, int shares, const void* ya, const float* pa, int na, long long sa, \
                                        const float* wa, float eps_a, float scale_a, const void* yb,              \
                                        const float* pb, int nb, long long sb, const float* wb, float eps_b,      \
                                        float scale_b, const float* w, const float* bias, void* out,              \
                                        const int* rows, int n_out, int hidden, float eps, int vec, void* stream) { \
    return add_layernorm_entry<T>(h, shares, LnShare<T>{(const T*)ya, pa, na, sa, wa, eps_a, scale_a},            \
                                  LnShare<T>{(const T*)yb, pb, nb, sb, wb, eps_b, scale_b}, w, bias, (T*)out,     \
                                  rows, n_out, hidden, eps, vec, stream);                                         \
  }

DEFINE_LAYER_NORM(bf16, bf16_t)
DEFINE_LAYER_NORM(f32, float)
