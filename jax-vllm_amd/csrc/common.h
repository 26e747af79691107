// Shared device helpers for the gfx950 (CDNA4, wave64) kernels of this library.
//
// Conventions of every exported entry point (extern "C", prefix jv_):
//   * raw device pointers, sizes as int / long long, the HIP stream last as void*;
//   * returns the hipError_t of the launch as int (0 = success), launches nothing
//     when a size is zero, and allocates nothing;
//   * element types: "bf16" entry points take __bf16 activations and weights,
//     "f32" entry points take float; reductions, softmax, norms and rotation
//     angles are float in both.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

#define JV_WAVE 64

typedef __bf16 bf16_t;

template <typename T> __device__ __forceinline__ float to_f32(T x) { return (float)x; }
template <typename T> __device__ __forceinline__ T from_f32(float x) { return (T)x; }

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = JV_WAVE / 2; o > 0; o >>= 1) v += __shfl_xor(v, o, JV_WAVE);
  return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int o = JV_WAVE / 2; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, JV_WAVE));
  return v;
}

// The maximum over a wave by moves between the lanes' registers (no LDS traffic): shifts inside the rows of 16 lanes, then
// the rows' last lanes broadcast into the next rows; lane 63 ends up with the whole wave's, NaNs are not seen.
template <int CTRL> __device__ __forceinline__ float lane_move(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(__float_as_int(v), __float_as_int(v), CTRL, 0xf, 0xf, false));
}
__device__ __forceinline__ float wave_max_lanes(float v) {
  v = fmaxf(v, lane_move<0x111>(v));      // row_shr:1, 2, 4, 8
  v = fmaxf(v, lane_move<0x112>(v));
  v = fmaxf(v, lane_move<0x114>(v));
  v = fmaxf(v, lane_move<0x118>(v));
  v = fmaxf(v, lane_move<0x142>(v));      // row_bcast:15
  v = fmaxf(v, lane_move<0x143>(v));      // row_bcast:31
  return __int_as_float(__builtin_amdgcn_readlane(__float_as_int(v), 63));
}

// Sum over a whole block of up to 1024 threads; `red` is shared scratch of >= 17 floats.
__device__ __forceinline__ float block_sum(float v, float* red) {
  const int lane = threadIdx.x & (JV_WAVE - 1), wid = threadIdx.x / JV_WAVE;
  const int nw = (blockDim.x + JV_WAVE - 1) / JV_WAVE;
  v = wave_sum(v);
  __syncthreads();  // protects `red` against a previous use
  if (lane == 0) red[wid] = v;
  __syncthreads();
  float t = (lane < nw) ? red[lane] : 0.f;
  t = wave_sum(t);
  return t;
}

// Gate activations of a gated feed-forward, y = act(gate) * up, in float.  The ids are part of the
// exported interface (the Python side names them).
#define JV_ACT_SILU 1        // gate / (1 + exp(-gate))
#define JV_ACT_GELU_TANH 2   // 0.5 gate (1 + tanh(sqrt(2/pi) (gate + 0.044715 gate^3)))
#define JV_ACT_CLAMPED 6     // g / (1 + exp(-slope g)) (u + 1) with g = min(gate, limit), u = up clamped to [-limit, limit]
// An activation with its constants (those of JV_ACT_CLAMPED; the others have none).
struct JvAct { int id; float limit, slope; };
__host__ __device__ __forceinline__ bool jv_act_known(int act) {
  return act == JV_ACT_SILU || act == JV_ACT_GELU_TANH || act == JV_ACT_CLAMPED;
}
__device__ __forceinline__ float jv_gated(JvAct act, float gate, float up) {
  if (act.id == JV_ACT_GELU_TANH) {
    const float inner = 0.7978845608028654f * (gate + 0.044715f * gate * gate * gate);
    return 0.5f * gate * (1.f + tanhf(inner)) * up;
  }
  if (act.id == JV_ACT_CLAMPED) {      // comparisons that a NaN passes through
    const float g = gate > act.limit ? act.limit : gate;
    const float u = up > act.limit ? act.limit : up < -act.limit ? -act.limit : up;
    return g / (1.f + expf(-act.slope * g)) * (u + 1.f);
  }
  return gate / (1.f + expf(-gate)) * up;
}

// Activations that stand alone (a feed-forward without a gate), in float; 0 means none.
#define JV_ACT_GELU_ERF 3    // 0.5 z (1 + erf(z / sqrt(2)))
#define JV_ACT_TANH 4
#define JV_ACT_RELU2 5       // max(z, 0)^2
__host__ __device__ __forceinline__ bool jv_plain_act_known(int act) { return act >= JV_ACT_SILU && act <= JV_ACT_RELU2; }
__device__ __forceinline__ float jv_act(int act, float z) {
  if (act == JV_ACT_GELU_ERF) return 0.5f * z * (1.f + erff(z * 0.7071067811865476f));
  if (act == JV_ACT_TANH) return tanhf(z);
  if (act == JV_ACT_RELU2) { const float p = fmaxf(z, 0.f); return z != z ? z : p * p; }
  if (act == JV_ACT_GELU_TANH) return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
  if (act == JV_ACT_SILU) return z / (1.f + expf(-z));
  return z;
}

// N consecutive floats (a multiple of 4) in pieces of 16 bytes, from any address of a float.
template <int N> __device__ __forceinline__ void load_floats(const float* p, float (&v)[N]) {
  typedef float f4 __attribute__((ext_vector_type(4), aligned(4)));
#pragma unroll
  for (int i = 0; i < N; i += 4) {
    const f4 x = *(const f4*)(p + i);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[i + e] = x[e];
  }
}

#define JV_LAUNCH_CHECK() ((int)hipGetLastError())
