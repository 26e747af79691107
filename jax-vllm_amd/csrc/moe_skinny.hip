// The two grouped products of routed experts for steps of few tokens (decode): every chosen expert has a row or a few,
// so the time is the reading of its weights.  bfloat16, float accumulation; the grouping they read has tiles of at most
// 16 rows of one expert.
//
// A block of 4 waves takes one tile of (token, choice) rows against 64 / WK rows of the expert's weight: WK waves share
// out the inner size of 16 rows of W (a long inner size gives every wave enough of it, a short one goes to one wave).  A
// wave streams its slice of W straight into MFMA operands (v_mfma_f32_16x16x32_bf16, A = 16 rows of W, B = the tile's
// rows of x: rows beyond the tile repeat its last one and cost no bytes), STEPS steps asked for while the ones before are
// multiplied.  W's addresses hang on the tile's expert alone, so its first loads are on their way while the chain
// offsets -> order -> rows of x is walked.  The waves' sums are added in LDS in their order: an output row is one fixed
// sum whatever else is in the step.
//   MS_GATED:  z[pos] = act(w g) * (w u), g = Wg[e] x[token], u = Wu[e] x[token]    (bf16)
//   MS_PLAIN:  z[pos] = act(w u), u = Wu[e] x[token]: experts without a gate        (bf16)
//   MS_DOWN:   y[kk][token] = (Wd[e] z[pos]) * w_out                                (float)
#include "common.h"

typedef __bf16 ms_bf16x8 __attribute__((ext_vector_type(8)));
typedef float ms_f32x4 __attribute__((ext_vector_type(4)));

enum { MS_DOWN = 0, MS_GATED = 1, MS_PLAIN = 2 };
#define MS_ROWS 16
#define MS_STEPS 2      // measured at 2,048 x 768 and 4,096 x 1,536, 8 tokens: 74 MB in 18.6 us and 440 MB in 79 us; 4 steps 21 and 81

template <int MODE, int WK>
__global__ void __launch_bounds__(256)
moe_skinny_kernel(void* __restrict__ out, const bf16_t* __restrict__ a_rows, const bf16_t* __restrict__ W0,
                  const bf16_t* __restrict__ W1, const int* __restrict__ meta, const int* __restrict__ offsets,
                  const int* __restrict__ tile_expert, const int* __restrict__ tile_row0, const int* __restrict__ order,
                  const float* __restrict__ weights, int top, int n_tokens, int K, int N, JvAct act, int use_weight) {
  constexpr bool GATED = MODE == MS_GATED, BY_TOKEN = MODE != MS_DOWN;
  constexpr int STEPS = MS_STEPS, NB = 64 / WK;          // rows of W a block takes
  __shared__ float red[GATED ? 2 : 1][4][16][17];
  // neighbouring blocks take neighbouring rows of one expert: what is read at one time lies side by side (blocks of
  // different experts at the same rows would be a whole expert apart, and meet on the same memory channels)
  const int per_tile = (N + NB - 1) / NB, tile = blockIdx.x / per_tile;
  const int tiles = meta[0], e = tile_expert[tile], row0 = tile_row0[tile];
  if (tile >= tiles) return;                             // (the entries beyond the tiles hold anything)
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, li = lane & 15, lc = lane >> 4;
  const int n0 = (blockIdx.x - tile * per_tile) * NB, wn = n0 + wave / WK * 16;
  const long long wr = ((long long)e * N + min(wn + li, N - 1)) * K;
  const bf16_t* w0 = W0 + wr;
  const bf16_t* w1 = GATED ? W1 + wr : W0;
  const int steps = (K + 31) / 32, per_wave = (steps + WK - 1) / WK;
  const int s_lo = wave % WK * per_wave, s_hi = min(steps, s_lo + per_wave);
  const ms_bf16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  ms_f32x4 acc0 = {0.f, 0.f, 0.f, 0.f}, acc1 = {0.f, 0.f, 0.f, 0.f};
  ms_bf16x8 a0[2][STEPS], a1[2][GATED ? STEPS : 1], b[2][STEPS];
  auto column = [&](int s) { return min(min(s, s_hi - 1) * 32 + lc * 8, K - 8); };   // beyond the slice: its last columns again
  auto fetch_w = [&](int buf, int s0) {
#pragma unroll
    for (int u = 0; u < STEPS; ++u) {
      a0[buf][u] = *(const ms_bf16x8*)(w0 + column(s0 + u));
      if (GATED) a1[buf][u] = *(const ms_bf16x8*)(w1 + column(s0 + u));
    }
  };
  const bool live = s_lo < s_hi && wn < N;
  if (live) fetch_w(0, s_lo);
  const int rows = min(MS_ROWS, offsets[e + 1] - row0);
  const int mine = row0 + min(li, rows - 1);
  const bf16_t* xr = a_rows + (BY_TOKEN ? (long long)(order[mine] / top) : (long long)mine) * K;
  auto fetch_x = [&](int buf, int s0) {
#pragma unroll
    for (int u = 0; u < STEPS; ++u) b[buf][u] = *(const ms_bf16x8*)(xr + column(s0 + u));
  };
  auto multiply = [&](int buf, int s0) {
#pragma unroll
    for (int u = 0; u < STEPS; ++u) {
      const bool in = s0 + u < s_hi && (s0 + u) * 32 + lc * 8 < K;
      const ms_bf16x8 x = in ? b[buf][u] : zero;
      acc0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a0[buf][u], x, acc0, 0, 0, 0);
      if (GATED) acc1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a1[buf][u], x, acc1, 0, 0, 0);
    }
  };
  if (live) {
    fetch_x(0, s_lo);
    for (int s = s_lo; s < s_hi; s += 2 * STEPS) {
      fetch_w(1, s + STEPS);
      fetch_x(1, s + STEPS);
      __builtin_amdgcn_sched_barrier(0);
      multiply(0, s);
      fetch_w(0, s + 2 * STEPS);
      fetch_x(0, s + 2 * STEPS);
      __builtin_amdgcn_sched_barrier(0);
      multiply(1, s + STEPS);
    }
  }
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    red[0][wave][lc * 4 + c][li] = acc0[c];
    if (GATED) red[GATED ? 1 : 0][wave][lc * 4 + c][li] = acc1[c];
  }
  __syncthreads();
  for (int i = tid; i < NB * 16; i += 256) {
    const int m = i / NB, nl = i - m * NB, n = n0 + nl;
    if (m >= rows || n >= N) continue;
    float y0 = 0.f, y1 = 0.f;                            // sums with W0 and, gated, with W1
#pragma unroll
    for (int ww = 0; ww < WK; ++ww) {
      y0 += red[0][nl / 16 * WK + ww][nl & 15][m];
      if (GATED) y1 += red[GATED ? 1 : 0][nl / 16 * WK + ww][nl & 15][m];
    }
    const int s = order[row0 + m];
    const float w = use_weight ? weights[s] : 1.f;
    if (MODE == MS_GATED) {
      ((bf16_t*)out)[(long long)(row0 + m) * N + n] = from_f32<bf16_t>(jv_gated(act, y0 * w, y1 * w));
    } else if (MODE == MS_PLAIN) {
      ((bf16_t*)out)[(long long)(row0 + m) * N + n] = from_f32<bf16_t>(jv_act(act.id, y0 * w));
    } else {
      const int token = s / top, kk = s - token * top;
      ((float*)out)[((long long)kk * n_tokens + token) * N + n] = y0 * w;
    }
  }
}

template <int MODE>
static int launch_moe_skinny(void* out, const void* a, const void* W0, const void* W1, const int* meta, const int* offsets,
                             const int* tile_expert, const int* tile_row0, const int* order, const float* weights,
                             int max_tiles, int top, int n_tokens, int K, int N, JvAct act, int use_weight, void* stream) {
  if (K < 8 || K % 8) return (int)hipErrorInvalidValue;
  const int wk = K >= 2048 ? 4 : 2;
  auto kernel = wk == 4 ? moe_skinny_kernel<MODE, 4> : moe_skinny_kernel<MODE, 2>;
  const int nb = 64 / wk;
  const long long blocks = (long long)max_tiles * ((N + nb - 1) / nb);
  if (blocks > 0x7fffffffll) return (int)hipErrorInvalidValue;
  hipLaunchKernelGGL(kernel, dim3((unsigned)blocks), dim3(256), 0, (hipStream_t)stream, out, (const bf16_t*)a,
                     (const bf16_t*)W0, (const bf16_t*)W1, meta, offsets, tile_expert, tile_row0, order, weights, top,
                     n_tokens, K, N, act, use_weight);
  return JV_LAUNCH_CHECK();
}

extern "C" int jv_moe_skinny_rows() { return MS_ROWS; }

// gate/up: x [tokens, hidden], Wg, Wu [experts, ff, hidden] -> z [entries, ff] bf16 by position.  Wg null: experts
// without a gate, act one that stands alone.
extern "C" int jv_moe_gate_up_skinny_bf16(void* z, const void* x, const void* Wg, const void* Wu, const int* meta,
                                          const int* offsets, const int* tile_expert, const int* tile_row0,
                                          const int* order, const float* weights, int max_tiles, int top, int hidden,
                                          int ff, int act, float act_limit, float act_slope, int scale_input, void* stream) {
  if (max_tiles <= 0 || ff <= 0) return 0;
  if (!(Wg ? jv_act_known(act) : jv_plain_act_known(act))) return (int)hipErrorInvalidValue;
  if (Wg)
    return launch_moe_skinny<MS_GATED>(z, x, Wg, Wu, meta, offsets, tile_expert, tile_row0, order, weights, max_tiles, top,
                                       0, hidden, ff, JvAct{act, act_limit, act_slope}, scale_input, stream);
  return launch_moe_skinny<MS_PLAIN>(z, x, Wu, nullptr, meta, offsets, tile_expert, tile_row0, order, weights, max_tiles,
                                     top, 0, hidden, ff, JvAct{act, act_limit, act_slope}, scale_input, stream);
}

// down: z [entries, ff] by position, Wd [experts, hidden, ff] -> y [top, tokens, hidden] float
extern "C" int jv_moe_down_skinny_bf16(float* y, const void* z, const void* Wd, const int* meta, const int* offsets,
                                       const int* tile_expert, const int* tile_row0, const int* order,
                                       const float* weights, int max_tiles, int top, int n_tokens, int hidden, int ff,
                                       int scale_output, void* stream) {
  if (max_tiles <= 0 || hidden <= 0) return 0;
  return launch_moe_skinny<MS_DOWN>(y, z, Wd, nullptr, meta, offsets, tile_expert, tile_row0, order, weights, max_tiles,
                                    top, n_tokens, ff, hidden, JvAct{}, scale_output, stream);
}
