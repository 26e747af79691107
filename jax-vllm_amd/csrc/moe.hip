// Routed experts: choice of experts per token, rows grouped by expert on the device, and the two
// grouped matrix products of gated experts.  Nothing here returns to the host: a step's routing is
// known only on the device, so every launch is sized by upper bounds and blocks without work leave.
//
//   route:   z = router logits (float, plus an optional bias per expert) -> the `top` largest per token
//            (lowest index among equals), weight = sigmoid(z), or the softmax over the chosen logits alone, or
//            ("sigmoid_normed") the largest sigmoid(z) + correction chosen, weight = sigmoid(z) over the sum of the
//            chosen sigmoids (+ 1e-20) times a constant, or ("sigmoid_corrected") chosen alike, weight = sigmoid(z) times a
//            constant, or ("softmax") the softmax over ALL logits, as it is.
//            Experts may form equal groups of neighbours: only those of the `keep` groups with the largest logits
//            (lowest group among equals) can then be chosen
//   group:   entry s = token * top + kk  ->  position in a list ordered by expert; tiles of MOE_TM rows
//            that never straddle two experts
//   gate/up: z[pos] = act(w g) * (w u),  g = Wg[e] x[token], u = Wu[e] x[token]      (w = the entry's weight
//            when it scales the expert's INPUT: w (W x) = W (w x); else 1); experts without a gate: act(w u)
//   down:    y[kk][token] = (Wd[e] z[pos]) * (w if it scales the OUTPUT else 1)        float
// The order of rows inside an expert's group depends on timing; no result does: every output row is a
// sum over the inner size in ascending order, alone.
#include "common.h"

#define MOE_TM 64
#define MOE_TN 64
#define MOE_BK 16

// The `top` largest of a token's logits, lowest index among equals: the lanes of a wave scan the token's
// logits (a copy in LDS), the wave agrees on the best, and the lane that scans the chosen expert takes it out.
#define MOE_SCORE_SIGMOID 0          // weight = sigmoid(logit)
#define MOE_SCORE_SOFTMAX_CHOSEN 1   // weight = exp(logit) / sum of exp over the token's chosen logits
#define MOE_SCORE_SIGMOID_NORMED 2   // chosen by sigmoid(logit) + correction; weight = sigmoid(logit) / (sum over the chosen + 1e-20) * scale
#define MOE_SCORE_SOFTMAX 3          // weight = exp(logit) / sum of exp over all of the token's logits
#define MOE_SCORE_SIGMOID_CORRECTED 4  // chosen by sigmoid(logit) + correction; weight = sigmoid(logit) * scale
#define MOE_SCORE_LAST 4
#define MOE_MAX_GROUPS 64
#define MOE_LANE_EXPERTS 256         // up to so many experts a lane keeps its own in registers
__device__ __forceinline__ void moe_pick(float* zt, int experts, int top, int lane, int* ids, float* weights,
                                         int score, const float* __restrict__ correction, float weight_scale,
                                         int groups, int keep) {
  const bool normed = score == MOE_SCORE_SIGMOID_NORMED;
  const bool corrected = normed || score == MOE_SCORE_SIGMOID_CORRECTED;      // the choice looks at sigmoid + correction
  float zmax = 0.f, inv_sum = 0.f;
  if (score == MOE_SCORE_SOFTMAX) {      // over all experts, before any is left out
    float m = -INFINITY, sum = 0.f;
    for (int e = lane; e < experts; e += JV_WAVE) m = fmaxf(m, zt[e]);
    zmax = wave_max(m);
    for (int e = lane; e < experts; e += JV_WAVE) sum += expf(zt[e] - zmax);
    inv_sum = 1.f / wave_sum(sum);
  }
  if (groups > 1 && keep < groups) {
    // lane g ranks group g by its largest logit; every lane then takes the lost groups' experts out of those it scans
    const int size = experts / groups;
    float best = -INFINITY;
    if (lane < groups)
      for (int i = 0; i < size; ++i) best = fmaxf(best, zt[lane * size + i]);
    int ahead = 0;
    for (int g = 0; g < groups; ++g) {
      const float other = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(best), g));
      if (other > best || (other == best && g < lane)) ++ahead;
    }
    const unsigned long long kept = __ballot(lane < groups && ahead < keep);
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");      // the groups are read before their entries change
    for (int e = lane; e < experts; e += JV_WAVE)
      if (!((kept >> (e / size)) & 1)) zt[e] = -INFINITY;
  }
  if (experts <= MOE_LANE_EXPERTS && top <= JV_WAVE) {
    // the values stay in registers; per choice one maximum across the wave by lane moves within the registers' rows, and
    // the lowest lane that holds it (the experts of the first 64 first); a taken expert becomes a NaN, which no maximum sees
    constexpr int PER = MOE_LANE_EXPERTS / JV_WAVE;
    float z[PER], c[PER];
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int e = lane + i * JV_WAVE;
      z[i] = e < experts ? zt[e] : 0.f;
      c[i] = z[i];
      if (corrected && z[i] != -INFINITY && e < experts) c[i] = 1.f / (1.f + expf(-z[i])) + (correction ? correction[e] : 0.f);
      if (c[i] != c[i]) c[i] = -INFINITY;         // a NaN takes the last places, its weight shows it
      if (e >= experts) c[i] = __builtin_nanf("");
    }
    float zk = 0.f;                               // of the lane's choice: lane kk keeps the kk-th
    int ek = 0;
    for (int kk = 0; kk < top; ++kk) {
      float m = c[0];
#pragma unroll
      for (int i = 1; i < PER; ++i) m = fmaxf(m, c[i]);
      m = wave_max_lanes(m);
      bool found = false;
#pragma unroll
      for (int i = 0; i < PER; ++i) {
        const unsigned long long at = __ballot(c[i] == m);
        if (found || !at) continue;
        found = true;
        const int l = __ffsll(at) - 1;
        const float zv = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(z[i]), l));
        if (lane == kk) { zk = zv; ek = l + i * JV_WAVE; }
        if (lane == l) c[i] = __builtin_nanf("");
      }
    }
    const bool mine = lane < top;
    float w;
    if (score == MOE_SCORE_SOFTMAX) {
      w = expf(zk - zmax) * inv_sum;
    } else if (score == MOE_SCORE_SOFTMAX_CHOSEN) {
      const float first = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(zk), 0));      // the largest
      w = mine ? expf(zk - first) : 0.f;
      w *= 1.f / wave_sum(w);
    } else {
      w = mine ? 1.f / (1.f + expf(-zk)) : 0.f;
      if (normed) w *= weight_scale / (wave_sum(w) + 1e-20f);
      else if (corrected) w *= weight_scale;
    }
    if (mine) {
      ids[lane] = ek;
      weights[lane] = w;
    }
    return;
  }
  for (int kk = 0; kk < top; ++kk) {
    float bv = -INFINITY;
    int bi = 0x7fffffff;
    for (int e = lane; e < experts; e += JV_WAVE) {
      float v = zt[e];
      // an expert already taken holds -inf and stays out; the others compete with their corrected sigmoid
      if (corrected && v != -INFINITY) v = 1.f / (1.f + expf(-v)) + (correction ? correction[e] : 0.f);
      if (v > bv || (bi == 0x7fffffff && v == v)) { bv = v; bi = e; }
    }
#pragma unroll
    for (int o = JV_WAVE / 2; o > 0; o >>= 1) {
      const float ov = __shfl_xor(bv, o, JV_WAVE);
      const int oi = __shfl_xor(bi, o, JV_WAVE);
      if (oi != 0x7fffffff && (bi == 0x7fffffff || ov > bv || (ov == bv && oi < bi))) { bv = ov; bi = oi; }
    }
    if (bi == 0x7fffffff) { bi = kk; bv = __builtin_nanf(""); }      // a row of NaN: some expert, the NaN shows in the output
    if (lane == 0) {
      ids[kk] = bi;
      const float z = corrected ? zt[bi] : bv;          // the logit itself: the correction takes part in the choice only
      weights[kk] = score == MOE_SCORE_SOFTMAX_CHOSEN ? bv : score == MOE_SCORE_SOFTMAX ? expf(z - zmax) * inv_sum
                                                                                        : 1.f / (1.f + expf(-z));
    }
    if ((bi & (JV_WAVE - 1)) == lane) zt[bi] = -INFINITY;
  }
  if (score == MOE_SCORE_SOFTMAX_CHOSEN && lane == 0) {
    // the chosen logits came in descending order: the first is their maximum; sums in that order
    const float m = weights[0];
    float sum = 0.f;
    for (int kk = 0; kk < top; ++kk) {
      const float p = expf(weights[kk] - m);
      weights[kk] = p;
      sum += p;
    }
    const float inv = 1.f / sum;
    for (int kk = 0; kk < top; ++kk) weights[kk] *= inv;
  }
  if (corrected && !normed && lane == 0)
    for (int kk = 0; kk < top; ++kk) weights[kk] *= weight_scale;
  if (normed && lane == 0) {
    float sum = 0.f;
    for (int kk = 0; kk < top; ++kk) sum += weights[kk];
    const float f = weight_scale / (sum + 1e-20f);
    for (int kk = 0; kk < top; ++kk) weights[kk] *= f;
  }
}

// a wave per token, 4 tokens a block
__global__ void __launch_bounds__(256)
moe_route_kernel(const float* __restrict__ logits, const float* __restrict__ bias, int n, int experts, int top,
                 int score, int* __restrict__ ids, float* __restrict__ weights, const float* __restrict__ correction,
                 float weight_scale, int groups, int keep) {
  extern __shared__ float zs[];      // [4][experts]
  const int lane = threadIdx.x & (JV_WAVE - 1), wid = threadIdx.x / JV_WAVE;
  const long long t = (long long)blockIdx.x * 4 + wid;
  if (t >= n) return;
  float* zt = zs + wid * experts;
  for (int e = lane; e < experts; e += JV_WAVE) zt[e] = logits[t * experts + e] + (bias ? bias[e] : 0.f);
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");        // a group's lane reads what other lanes wrote
  moe_pick(zt, experts, top, lane, ids + t * top, weights + t * top, score, correction, weight_scale, groups, keep);
}

// Router and choice in one launch: a block takes up to MOE_RT tokens, their rows in LDS as floats; a wave per
// expert (in turns) reads the expert's router row once and sums its products with every token of the block
// lane by lane and then across the wave: float logits whatever the activation type, the same order of
// additions whatever the batch.  Then a wave per token picks the `top` largest, lowest index among equals.
// logits_out (may be null) [n, experts].
#define MOE_RT 8
template <typename T>
__global__ void __launch_bounds__(1024)
moe_router_kernel(const T* __restrict__ x, const T* __restrict__ W, const float* __restrict__ bias, int n, int hidden,
                  int experts, int top, int tb, int score, int* __restrict__ ids, float* __restrict__ weights,
                  float* __restrict__ logits_out, const float* __restrict__ correction, float weight_scale, int groups,
                  int keep) {
  extern __shared__ float rs[];      // x [tb][hidden] | z [tb][experts]
  float* xs = rs;
  float* z = rs + tb * hidden;
  const long long t0 = (long long)blockIdx.x * tb;
  const int nt = (int)min((long long)tb, n - t0);
  const int lane = threadIdx.x & (JV_WAVE - 1), wid = threadIdx.x / JV_WAVE, nw = blockDim.x / JV_WAVE;
  for (int i = threadIdx.x; i < tb * hidden; i += blockDim.x) {
    const int t = i / hidden;
    xs[i] = t < nt ? to_f32(x[t0 * hidden + i]) : 0.f;
  }
  __syncthreads();
  for (int e = wid; e < experts; e += nw) {
    const T* w = W + (long long)e * hidden;
    float acc[MOE_RT];
#pragma unroll
    for (int t = 0; t < MOE_RT; ++t) acc[t] = 0.f;
    // eight loads of the router row are asked for before their products: a wave's time here is its chain of loads
    for (int c0 = lane; c0 < hidden; c0 += 8 * JV_WAVE) {
      float wv[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const int c = c0 + u * JV_WAVE;
        wv[u] = to_f32(w[c < hidden ? c : lane]);
      }
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const int c = c0 + u * JV_WAVE;
        if (c < hidden) {
#pragma unroll
          for (int t = 0; t < MOE_RT; ++t)
            if (t < tb) acc[t] = fmaf(xs[t * hidden + c], wv[u], acc[t]);
        }
      }
    }
#pragma unroll
    for (int t = 0; t < MOE_RT; ++t) {
      if (t >= nt) continue;
      const float v = wave_sum(acc[t]) + (bias ? bias[e] : 0.f);
      if (lane == 0) {
        z[t * experts + e] = v;
        if (logits_out) logits_out[(t0 + t) * experts + e] = v;
      }
    }
  }
  __syncthreads();
  for (int t = wid; t < nt; t += nw)
    moe_pick(z + t * experts, experts, top, lane, ids + (t0 + t) * top, weights + (t0 + t) * top, score, correction,
             weight_scale, groups, keep);
}

// Exclusive sums over the experts of their entries and of their tiles, by one wave: start, tile0 [experts + 1].
__device__ __forceinline__ void moe_scan_counts(const int* count, int* start, int* tile0, int experts, int tile_rows, int lane) {
  int at = 0, tiles = 0;
  for (int e0 = 0; e0 < experts; e0 += JV_WAVE) {
    const int e = e0 + lane;
    const int c = e < experts ? count[e] : 0, t = (c + tile_rows - 1) / tile_rows;
    int ci = c, ti = t;
#pragma unroll
    for (int o = 1; o < JV_WAVE; o <<= 1) {
      const int cu = __shfl_up(ci, o, JV_WAVE), tu = __shfl_up(ti, o, JV_WAVE);
      if (lane >= o) { ci += cu; ti += tu; }
    }
    if (e < experts) { start[e] = at + ci - c; tile0[e] = tiles + ti - t; }
    at += __shfl(ci, JV_WAVE - 1, JV_WAVE);
    tiles += __shfl(ti, JV_WAVE - 1, JV_WAVE);
  }
  if (lane == 0) { start[experts] = at; tile0[experts] = tiles; }
}

// What a grouping hands on, from the sums: meta [0] number of tiles, offsets [experts + 1], tile_expert / tile_row0.
__device__ __forceinline__ void moe_write_tiles(const int* start, const int* tile0, int experts, int tile_rows, int* meta,
                                                int* offsets, int* tile_expert, int* tile_row0) {
  if (threadIdx.x == 0) meta[0] = tile0[experts];
  for (int e = threadIdx.x; e <= experts; e += blockDim.x) offsets[e] = start[e];
  for (int e = threadIdx.x; e < experts; e += blockDim.x)
    for (int i = tile0[e]; i < tile0[e + 1]; ++i) {
      tile_expert[i] = e;
      tile_row0[i] = start[e] + (i - tile0[e]) * tile_rows;
    }
}

// One block.  meta: [0] number of tiles; offsets [experts + 1]; tile_expert / tile_row0 [max_tiles];
// order [entries]: entry index at each position; rank [entries] scratch.  A tile has tile_rows rows.
__global__ void __launch_bounds__(1024)
moe_group_kernel(const int* __restrict__ ids, int entries, int experts, int tile_rows, int* __restrict__ meta,
                 int* __restrict__ offsets, int* __restrict__ tile_expert, int* __restrict__ tile_row0,
                 int* __restrict__ order, int* __restrict__ rank) {
  extern __shared__ int sh[];      // count [experts] | start [experts + 1] | first tile [experts + 1]
  int* count = sh;
  int* start = sh + experts;
  int* tile0 = start + experts + 1;
  for (int e = threadIdx.x; e < experts; e += blockDim.x) count[e] = 0;
  __syncthreads();
  for (int s = threadIdx.x; s < entries; s += blockDim.x) rank[s] = atomicAdd(&count[ids[s]], 1);
  __syncthreads();
  if (threadIdx.x < JV_WAVE) moe_scan_counts(count, start, tile0, experts, tile_rows, threadIdx.x);
  __syncthreads();
  moe_write_tiles(start, tile0, experts, tile_rows, meta, offsets, tile_expert, tile_row0);
  for (int s = threadIdx.x; s < entries; s += blockDim.x) order[start[ids[s]] + rank[s]] = s;
}

// Choice and grouping of few tokens in one launch of one block: a wave a token picks, then the block groups.  Every
// token has `top` chosen entries and `always` further ones, for the experts behind the routed ones (number experts,
// experts + 1, ...), whose weight is 1: a shared expert cut into pieces of the routed ones' size.  Entry s = token *
// (top + always) + kk.  The logits may come as `parts` partial products, added here in their order.  LDS: logits [16][experts] | ids [entries] | rank [entries] | count, start, first tile of experts + always.
__global__ void __launch_bounds__(1024)
moe_route_group_kernel(const float* __restrict__ logits, int parts, long long part_stride,
                       const float* __restrict__ bias, int n, int experts, int top, int always, int score, int* __restrict__ ids, float* __restrict__ weights,
                       const float* __restrict__ correction, float weight_scale, int groups, int keep, int tile_rows,
                       int* __restrict__ meta, int* __restrict__ offsets, int* __restrict__ tile_expert,
                       int* __restrict__ tile_row0, int* __restrict__ order) {
  extern __shared__ float zs[];
  const int all = experts + always, per = top + always, entries = n * per;
  int* lid = (int*)(zs + 16 * experts);
  int* rank = lid + entries;
  int* count = rank + entries;
  int* start = count + all;
  int* tile0 = start + all + 1;
  const int lane = threadIdx.x & (JV_WAVE - 1), wid = threadIdx.x / JV_WAVE, waves = blockDim.x / JV_WAVE;
  for (int e = threadIdx.x; e < all; e += blockDim.x) count[e] = 0;
  float* zt = zs + wid * experts;
  for (int t = wid; t < n; t += waves) {
    for (int e = lane; e < experts; e += JV_WAVE) {
      const float* at = logits + (long long)t * experts + e;
      float z = 0.f;
      for (int p0 = 0; p0 < parts; p0 += 8) {                     // eight asked for before they are added
        float v[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) v[u] = at[min(p0 + u, parts - 1) * part_stride];
#pragma unroll
        for (int u = 0; u < 8; ++u) z += p0 + u < parts ? v[u] : 0.f;
      }
      zt[e] = z + (bias ? bias[e] : 0.f);
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");        // a group's lane reads what other lanes wrote
    moe_pick(zt, experts, top, lane, lid + t * per, weights + (long long)t * per, score, correction, weight_scale, groups, keep);
    if (lane < always) {
      lid[t * per + top + lane] = experts + lane;
      weights[(long long)t * per + top + lane] = 1.f;
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");        // before the wave's next token takes its place
  }
  __syncthreads();
  for (int s = threadIdx.x; s < entries; s += blockDim.x) {
    const int e = lid[s];
    ids[s] = e;
    rank[s] = atomicAdd(&count[e], 1);
  }
  __syncthreads();
  if (wid == 0) moe_scan_counts(count, start, tile0, all, tile_rows, lane);
  __syncthreads();
  moe_write_tiles(start, tile0, all, tile_rows, meta, offsets, tile_expert, tile_row0);
  for (int s = threadIdx.x; s < entries; s += blockDim.x) order[start[lid[s]] + rank[s]] = s;
}

// grid (max tiles, column tiles of the expert width).  x [tokens, hidden]; Wg, Wu [experts, ff, hidden];
// z [entries, ff] by position.  Without GATED there is no Wg and the activation stands alone.
template <typename T, bool GATED>
__global__ void __launch_bounds__(256)
moe_gate_up_kernel(T* __restrict__ z, const T* __restrict__ x, const T* __restrict__ Wg, const T* __restrict__ Wu,
                   const int* __restrict__ meta, const int* __restrict__ offsets, const int* __restrict__ tile_expert,
                   const int* __restrict__ tile_row0, const int* __restrict__ order, const float* __restrict__ weights,
                   int top, int hidden, int ff, JvAct act, int scale_input) {
  if ((int)blockIdx.x >= meta[0]) return;
  __shared__ float As[MOE_BK][MOE_TM + 4];
  __shared__ float Gs[GATED ? MOE_BK : 1][MOE_TN + 4];
  __shared__ float Us[MOE_BK][MOE_TN + 4];
  __shared__ int tok[MOE_TM];
  __shared__ float wgt[MOE_TM];
  const int e = tile_expert[blockIdx.x], row0 = tile_row0[blockIdx.x];
  const int rows = min(MOE_TM, offsets[e + 1] - row0);
  const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
  const int n0 = blockIdx.y * MOE_TN;
  if (tid < MOE_TM) {
    const int s = tid < rows ? order[row0 + tid] : -1;
    tok[tid] = s < 0 ? -1 : s / top;
    wgt[tid] = (s < 0 || !scale_input) ? 1.f : weights[s];
  }
  __syncthreads();
  const T* G = GATED ? Wg + (long long)e * ff * hidden : nullptr;
  const T* U = Wu + (long long)e * ff * hidden;
  float ag[4][4] = {}, au[4][4] = {};
  for (int k0 = 0; k0 < hidden; k0 += MOE_BK) {
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const int idx = tid + q * 256;
      const int r = idx >> 4, kk = idx & 15, k = k0 + kk;
      const int tk = tok[r], wn = n0 + r;
      As[kk][r] = (tk >= 0 && k < hidden) ? to_f32(x[(long long)tk * hidden + k]) : 0.f;
      const bool in = wn < ff && k < hidden;
      if (GATED) Gs[kk][r] = in ? to_f32(G[(long long)wn * hidden + k]) : 0.f;
      Us[kk][r] = in ? to_f32(U[(long long)wn * hidden + k]) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < MOE_BK; ++kk) {
      float a[4], g[4], u[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) a[i] = As[kk][ty * 4 + i];
#pragma unroll
      for (int j = 0; j < 4; ++j) { g[j] = GATED ? Gs[GATED ? kk : 0][tx * 4 + j] : 0.f; u[j] = Us[kk][tx * 4 + j]; }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          if (GATED) ag[i][j] = fmaf(a[i], g[j], ag[i][j]);
          au[i][j] = fmaf(a[i], u[j], au[i][j]);
        }
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int m = ty * 4 + i;
    if (m >= rows) continue;
    const float w = wgt[m];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int n = n0 + tx * 4 + j;
      if (n < ff) z[(long long)(row0 + m) * ff + n] = from_f32<T>(GATED ? jv_gated(act, ag[i][j] * w, au[i][j] * w) : jv_act(act.id, au[i][j] * w));
    }
  }
}

// grid (max tiles, column tiles of hidden).  z [entries, ff] by position; Wd [experts, hidden, ff];
// y [top, tokens, hidden] float.
template <typename T>
__global__ void __launch_bounds__(256)
moe_down_kernel(float* __restrict__ y, const T* __restrict__ z, const T* __restrict__ Wd, const int* __restrict__ meta,
                const int* __restrict__ offsets, const int* __restrict__ tile_expert, const int* __restrict__ tile_row0,
                const int* __restrict__ order, const float* __restrict__ weights, int top, int n_tokens, int hidden,
                int ff, int scale_output) {
  if ((int)blockIdx.x >= meta[0]) return;
  __shared__ float As[MOE_BK][MOE_TM + 4];
  __shared__ float Ws[MOE_BK][MOE_TN + 4];
  __shared__ int ent[MOE_TM];
  const int e = tile_expert[blockIdx.x], row0 = tile_row0[blockIdx.x];
  const int rows = min(MOE_TM, offsets[e + 1] - row0);
  const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
  const int n0 = blockIdx.y * MOE_TN;
  if (tid < MOE_TM) ent[tid] = tid < rows ? order[row0 + tid] : -1;
  __syncthreads();
  const T* W = Wd + (long long)e * hidden * ff;
  float acc[4][4] = {};
  for (int k0 = 0; k0 < ff; k0 += MOE_BK) {
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const int idx = tid + q * 256;
      const int r = idx >> 4, kk = idx & 15, k = k0 + kk;
      const int wn = n0 + r;
      As[kk][r] = (r < rows && k < ff) ? to_f32(z[(long long)(row0 + r) * ff + k]) : 0.f;
      Ws[kk][r] = (wn < hidden && k < ff) ? to_f32(W[(long long)wn * ff + k]) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < MOE_BK; ++kk) {
      float a[4], b[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) a[i] = As[kk][ty * 4 + i];
#pragma unroll
      for (int j = 0; j < 4; ++j) b[j] = Ws[kk][tx * 4 + j];
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(a[i], b[j], acc[i][j]);
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int m = ty * 4 + i;
    if (m >= rows) continue;
    const int s = ent[m];
    const int token = s / top, kk = s - token * top;
    const float w = scale_output ? weights[s] : 1.f;
    float* o = y + ((long long)kk * n_tokens + token) * hidden;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int n = n0 + tx * 4 + j;
      if (n < hidden) o[n] = acc[i][j] * w;
    }
  }
}

// A share of every token that carries a gate of the token's own: out[t][c] = float(y[t][c]) * sigmoid(g[t * ldg])
// (a shared expert that joins the chosen experts' float stack under one number per token).
template <typename T>
__global__ void __launch_bounds__(256)
row_gate_kernel(float* __restrict__ out, const T* __restrict__ y, const T* __restrict__ g, long long ldg, long long n,
                int hidden) {
  const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= n * hidden) return;
  const long long t = i / hidden;
  out[i] = to_f32(y[i]) / (1.f + expf(-to_f32(g[t * ldg])));
}

// The same with four columns a lane, where the width and the addresses allow it.
template <typename T>
__global__ void __launch_bounds__(256)
row_gate_vec_kernel(float* __restrict__ out, const T* __restrict__ y, const T* __restrict__ g, long long ldg, long long n,
                    int hidden) {
  typedef T t4 __attribute__((ext_vector_type(4)));
  const long long i = ((long long)blockIdx.x * blockDim.x + threadIdx.x) * 4;
  if (i >= n * hidden) return;
  const long long t = i / hidden;
  const float gate = 1.f / (1.f + expf(-to_f32(g[t * ldg])));
  const t4 v = *(const t4*)(y + i);
  *(float4*)(out + i) = float4{to_f32(v[0]) * gate, to_f32(v[1]) * gate, to_f32(v[2]) * gate, to_f32(v[3]) * gate};
}

extern "C" int jv_moe_tile_rows() { return MOE_TM; }

// equal groups of neighbours, the kept ones with enough experts for the choice (groups <= 1: none)
static bool moe_groups_ok(int experts, int top, int groups, int keep) {
  return groups <= 1 || (groups <= MOE_MAX_GROUPS && experts % groups == 0 && keep >= 1 && keep <= groups &&
                         (long long)keep * (experts / groups) >= top);
}

extern "C" int jv_moe_route(const float* logits, const float* bias, int n, int experts, int top, int score, int* ids,
                            float* weights, const float* correction, float weight_scale, int groups, int keep,
                            void* stream) {
  if (n <= 0) return 0;
  if (experts <= 0 || top <= 0 || top > experts || score < 0 || score > MOE_SCORE_LAST)
    return (int)hipErrorInvalidValue;
  if (!moe_groups_ok(experts, top, groups, keep)) return (int)hipErrorInvalidValue;
  if (experts > 3840) return (int)hipErrorInvalidValue;
  hipLaunchKernelGGL(moe_route_kernel, dim3((n + 3) / 4), dim3(256), 4 * experts * sizeof(float), (hipStream_t)stream,
                     logits, bias, n, experts, top, score, ids, weights, correction, weight_scale, groups, keep);
  return JV_LAUNCH_CHECK();
}

// 1 if the one-block form takes these sizes, else 0
extern "C" int jv_moe_route_group_fits(int n, int experts, int top, int always) {
  if (n <= 0 || experts <= 0 || top <= 0 || always < 0 || always > JV_WAVE) return 0;
  return n <= 64 && (16LL * experts + 2LL * n * (top + always) + 3LL * (experts + always) + 2) * 4 <= 60 * 1024;
}

extern "C" int jv_moe_route_group(const float* logits, int parts, long long part_stride, const float* bias, int n, int experts, int top, int always, int score,
                                  int* ids, float* weights, const float* correction, float weight_scale, int groups,
                                  int keep, int tile_rows, int* meta, int* offsets, int* tile_expert, int* tile_row0,
                                  int* order, void* stream) {
  if (n <= 0) return 0;
  if (!jv_moe_route_group_fits(n, experts, top, always) || top > experts || score < 0 || score > MOE_SCORE_LAST ||
      !moe_groups_ok(experts, top, groups, keep) || tile_rows <= 0 || parts < 1)
    return (int)hipErrorInvalidValue;
  const size_t shmem = (16 * (size_t)experts + 2 * (size_t)n * (top + always) + 3 * (size_t)(experts + always) + 2) * 4;
  const int waves = n < 4 ? 4 : n > 16 ? 16 : n;
  hipLaunchKernelGGL(moe_route_group_kernel, dim3(1), dim3(64 * waves), shmem, (hipStream_t)stream, logits, parts,
                     part_stride, bias, n, experts, top, always, score, ids, weights, correction, weight_scale, groups, keep, tile_rows, meta, offsets,
                     tile_expert, tile_row0, order);
  return JV_LAUNCH_CHECK();
}

extern "C" int jv_moe_group(const int* ids, int entries, int experts, int tile_rows, int* meta, int* offsets,
                            int* tile_expert, int* tile_row0, int* order, int* rank, void* stream) {
  if (entries <= 0) return 0;
  if (experts <= 0 || experts > 4096 || tile_rows <= 0) return (int)hipErrorInvalidValue;
  hipLaunchKernelGGL(moe_group_kernel, dim3(1), dim3(1024), (3 * experts + 2) * sizeof(int), (hipStream_t)stream, ids,
                     entries, experts, tile_rows, meta, offsets, tile_expert, tile_row0, order, rank);
  return JV_LAUNCH_CHECK();
}

#define DEFINE_MOE(SUF, T)                                                                                        \
  extern "C" int jv_moe_router_##SUF(const void* x, const void* W, const float* bias, int n, int hidden,          \
                                     int experts, int top, int score, int* ids, float* weights,                   \
                                     float* logits_out, const float* correction, float weight_scale, int groups,  \
                                     int keep, void* stream) {                                                    \
    if (n <= 0) return 0;                                                                                         \
    if (experts <= 0 || top <= 0 || top > experts || hidden <= 0 || (hidden + experts) > 15000 || score < 0 ||    \
        score > MOE_SCORE_LAST || !moe_groups_ok(experts, top, groups, keep))                                  \
      return (int)hipErrorInvalidValue;                                                                           \
    int tb = 15000 / (hidden + experts);             /* tokens of a block: their rows and logits in 60 KB */      \
    tb = tb > MOE_RT ? MOE_RT : tb;                                                                               \
    while (tb > 1 && (n + tb - 1) / tb < 128) --tb;  /* few tokens: more blocks rather than rows sharing a read */ \
    hipLaunchKernelGGL(moe_router_kernel<T>, dim3((n + tb - 1) / tb), dim3(1024),                                  \
                       (size_t)tb * (hidden + experts) * sizeof(float), (hipStream_t)stream, (const T*)x,         \
                       (const T*)W, bias, n, hidden, experts, top, tb, score, ids, weights, logits_out,           \
                       correction, weight_scale, groups, keep);                                                   \
    return JV_LAUNCH_CHECK();                                                                                     \
  }                                                                                                               \
  extern "C" int jv_row_gate_##SUF(float* out, const void* y, const void* g, long long ldg, long long n,         \
                                   int hidden, void* stream) {                                                    \
    if (n <= 0 || hidden <= 0) return 0;                                                                          \
    if ((n * hidden + 255) / 256 > 0x7fffffffll) return (int)hipErrorInvalidValue;                                \
    if (hidden % 4 == 0 && (uintptr_t)out % 16 == 0 && (uintptr_t)y % (4 * sizeof(T)) == 0) {                     \
      hipLaunchKernelGGL(row_gate_vec_kernel<T>, dim3((unsigned)((n * hidden / 4 + 255) / 256)), dim3(256), 0,    \
                         (hipStream_t)stream, out, (const T*)y, (const T*)g, ldg, n, hidden);                     \
      return JV_LAUNCH_CHECK();                                                                                   \
    }                                                                                                             \
    hipLaunchKernelGGL(row_gate_kernel<T>, dim3((unsigned)((n * hidden + 255) / 256)), dim3(256), 0,              \
                       (hipStream_t)stream, out, (const T*)y, (const T*)g, ldg, n, hidden);                       \
    return JV_LAUNCH_CHECK();                                                                                     \
  }                                                                                                               \
  extern "C" int jv_moe_gate_up_##SUF(void* z, const void* x, const void* Wg, const void* Wu, const int* meta,    \
                                      const int* offsets, const int* tile_expert, const int* tile_row0,           \
                                      const int* order, const float* weights, int max_tiles, int top, int hidden, \
                                      int ff, int act, float act_limit, float act_slope, int scale_input, void* stream) {                           \
    if (max_tiles <= 0 || ff <= 0) return 0;                                                                      \
    if (!(Wg ? jv_act_known(act) : jv_plain_act_known(act)) || (ff + MOE_TN - 1) / MOE_TN > 65535)                \
      return (int)hipErrorInvalidValue;                                                                           \
    auto kernel = Wg ? moe_gate_up_kernel<T, true> : moe_gate_up_kernel<T, false>;                                \
    hipLaunchKernelGGL(kernel, dim3(max_tiles, (ff + MOE_TN - 1) / MOE_TN), dim3(256), 0,          \
                       (hipStream_t)stream, (T*)z, (const T*)x, (const T*)Wg, (const T*)Wu, meta, offsets,        \
                       tile_expert, tile_row0, order, weights, top, hidden, ff, JvAct{act, act_limit, act_slope}, scale_input);                \
    return JV_LAUNCH_CHECK();                                                                                     \
  }                                                                                                               \
  extern "C" int jv_moe_down_##SUF(float* y, const void* z, const void* Wd, const int* meta, const int* offsets,  \
                                   const int* tile_expert, const int* tile_row0, const int* order,                \
                                   const float* weights, int max_tiles, int top, int n_tokens, int hidden,        \
                                   int ff, int scale_output, void* stream) {                                      \
    if (max_tiles <= 0 || hidden <= 0) return 0;                                                                  \
    if ((hidden + MOE_TN - 1) / MOE_TN > 65535) return (int)hipErrorInvalidValue;                                 \
    hipLaunchKernelGGL(moe_down_kernel<T>, dim3(max_tiles, (hidden + MOE_TN - 1) / MOE_TN), dim3(256), 0,         \
                       (hipStream_t)stream, y, (const T*)z, (const T*)Wd, meta, offsets, tile_expert, tile_row0,  \
                       order, weights, top, n_tokens, hidden, ff, scale_output);                                  \
    return JV_LAUNCH_CHECK();                                                                                     \
  }

DEFINE_MOE(bf16, bf16_t)
DEFINE_MOE(f32, float)
