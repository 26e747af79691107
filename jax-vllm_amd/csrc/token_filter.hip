// Short causal filters over time per channel, and the attention input and output that go with them.
//
//   token_filter            out[t] = x[t] + sum_lag w[lag] x[t - lag]   (a sublayer's input plus its filter)
//   attn_prepare_filtered   projected q, k, v -> filter -> rotation -> q rows and cache pages, v rotated as well
//   rotate_back_gate        attention output turned back by its own position, times sigmoid(gate)
//
// A request's last taps - 1 inputs live in its row of `state` [slots + 1][taps - 1][channels] (float; row j holds the
// input of lag taps - 1 - j, zeros before a sequence's start).  Filter weights come as [taps][channels] (row j weighs
// lag taps - 1 - j).  A thread takes E neighbouring channels of one request over a segment of tokens and keeps the
// last inputs in registers.  The thread of a request's first segment is the only one that reads the old state (a first
// segment holds more rows than a filter has lags, or all of the request's), and it leaves the new one.
#include "common.h"

#define TF_MAX_LAGS 7
#define TF_BYTES 8        // of neighbouring channels a thread takes (2,048 tokens, 16 + 2 * 4 heads of 128: 15.6 us, with 16 bytes 20.3)
#define TF_RUN 8          // rows a thread asks for at once; a segment of token_filter

template <typename T, int E> struct TfVec { typedef T type __attribute__((ext_vector_type(E))); };
template <typename T> struct TfVec<T, 1> { struct type { T v; __device__ T operator[](int) const { return v; } }; };

template <typename T, int E> __device__ __forceinline__ void tf_load(const T* p, float (&v)[E]) {
  if constexpr (E == 1) {
    v[0] = to_f32<T>(*p);
  } else {
    const typename TfVec<T, E>::type x = *(const typename TfVec<T, E>::type*)p;
#pragma unroll
    for (int e = 0; e < E; ++e) v[e] = to_f32<T>(x[e]);
  }
}
template <typename T, int E> __device__ __forceinline__ void tf_widen(const typename TfVec<T, E>::type& x, float (&v)[E]) {
#pragma unroll
  for (int e = 0; e < E; ++e) v[e] = to_f32<T>(x[e]);
}
template <typename T, int E> __device__ __forceinline__ void tf_store(T* p, const float (&v)[E]) {
  if constexpr (E == 1) {
    *p = from_f32<T>(v[0]);
  } else {
    typename TfVec<T, E>::type x;
#pragma unroll
    for (int e = 0; e < E; ++e) x[e] = from_f32<T>(v[e]);
    *(typename TfVec<T, E>::type*)p = x;
  }
}

// The window of the last L inputs and the weights of one thread's channels.  L is at least the filter's lags; lags the
// filter does not have weigh nothing.  `wt` null: the filter is the identity.
template <int E, int L> struct TfWindow {
  float win[L][E], wl[L][E], w0[E];

  template <typename T>
  __device__ __forceinline__ void open(const T* in, long long ld, int first, const float* st, int lags, int channels,
                                       const float* wt) {
#pragma unroll
    for (int p = 0; p < L; ++p) {
      const int lag = L - p;
#pragma unroll
      for (int e = 0; e < E; ++e) win[p][e] = wl[p][e] = 0.f;
      if (lag <= lags) {
        tf_load<float, E>(wt + (long long)(lags - lag) * channels, wl[p]);
        const int i = first - lag;
        if (i >= 0) tf_load<T, E>(in + (long long)i * ld, win[p]);
        else tf_load<float, E>(st + (long long)(lags + i) * channels, win[p]);
      }
    }
#pragma unroll
    for (int e = 0; e < E; ++e) w0[e] = 1.f;
    if (wt) tf_load<float, E>(wt + (long long)lags * channels, w0);
  }
  // the filter's value at the next input x, which then joins the window
  __device__ __forceinline__ void step(const float (&x)[E], float (&y)[E]) {
#pragma unroll
    for (int e = 0; e < E; ++e) {
      float acc = 0.f;
#pragma unroll
      for (int p = 0; p < L; ++p) acc = fmaf(wl[p][e], win[p][e], acc);
      y[e] = fmaf(w0[e], x[e], acc);
#pragma unroll
      for (int p = 0; p + 1 < L; ++p) win[p][e] = win[p + 1][e];
      win[L - 1][e] = x[e];
    }
  }
};

// the last `lags` inputs of a request of n tokens: rows of this step, or, for a short step, old state rows moved up
// (row j takes row j + n: read before any row above j is written)
template <typename T, int E>
__device__ __forceinline__ void tf_leave_state(const T* in, long long ld, int n, float* st, int lags, int channels) {
  for (int j = 0; j < lags; ++j) {
    const int i = n - lags + j;
    float v[E];
    if (i >= 0) tf_load<T, E>(in + (long long)i * ld, v);
    else tf_load<float, E>(st + (long long)(j + n) * channels, v);
    tf_store<float, E>(st + (long long)j * channels, v);
  }
}

// grid (requests, blocks of 256 pieces of E channels, segments of TF_RUN tokens)
template <typename T, int E, int L>
__global__ void __launch_bounds__(256)
token_filter_kernel(T* __restrict__ out, const T* __restrict__ x, int channels, int lags, const float* __restrict__ wt,
                    float* __restrict__ state, const int* __restrict__ slot_ids, const int* __restrict__ cu_seqlens) {
  const int r = blockIdx.x, c = (blockIdx.y * 256 + threadIdx.x) * E;
  if (c >= channels) return;
  const int t0 = cu_seqlens[r], n = cu_seqlens[r + 1] - t0;
  const int s0 = blockIdx.z * TF_RUN;
  if (s0 >= n) return;
  float* st = state + (long long)slot_ids[r] * lags * channels + c;
  const T* in = x + (long long)t0 * channels + c;
  T* o = out + (long long)t0 * channels + c;
  typename TfVec<T, E>::type raw[TF_RUN];
#pragma unroll
  for (int u = 0; u < TF_RUN; ++u) raw[u] = *(const typename TfVec<T, E>::type*)(in + (long long)min(s0 + u, n - 1) * channels);
  TfWindow<E, L> f;
  f.open(in, channels, s0, st, lags, channels, wt + c);
#pragma unroll
  for (int u = 0; u < TF_RUN; ++u) {
    if (s0 + u >= n) break;
    float a[E], y[E];
    tf_widen<T, E>(raw[u], a);
    f.step(a, y);
#pragma unroll
    for (int e = 0; e < E; ++e) y[e] += a[e];
    tf_store<T, E>(o + (long long)(s0 + u) * channels, y);
  }
  if (blockIdx.z == 0) tf_leave_state<T, E>(in, channels, n, st, lags, channels);
}

// ---------------------------------------------------------------- attention input
// A token's row begins with [q: nq * dk | k: nkv * dk | v: nkv * dv]; every channel goes through its filter, then
//   q, k: the pairs (2i, 2i + 1) of a head's first rot_dims elements turn by the token's angles k_cs [n][rot_dims]
//   v:    all pairs (2m, 2m + 1) turn by v_cs [n][dv]          (null: values as filtered)
// q goes to rows [n][nq][dp] (zeros behind dk), k to pages [page][nkv][slot][dp], v to transposed pages
// [page][nkv][dp][slot]; the pad of the pages is never written.  grid (requests, blocks of 256 pieces, segments):
// segments are cut at positions that are multiples of 8, so that 8 tokens of a value element that lie side by side in
// a page are written as one piece.  The first one has 16 positions (its first multiple of 8 may lie up to 7 before the
// step: 9 rows at least), the others 8.  ONE: a step of one token a request.
template <typename T> struct alignas(sizeof(T) * 8) TfPack8 { T v[8]; };

template <int E>
__device__ __forceinline__ void tf_turn(float (&y)[E], const float* cs, int half, int first, int dims) {
#pragma unroll
  for (int e = 0; e + 1 < E; e += 2) {
    const int m = (first + e) >> 1;
    if (first + e >= dims) break;
    const float c = cs[m], s = cs[half + m];
    const float a = y[e], b = y[e + 1];
    y[e] = a * c - b * s;
    y[e + 1] = b * c + a * s;
  }
}

template <typename T, int E, int L, bool ONE>
__global__ void __launch_bounds__(256)
attn_prepare_filtered_kernel(T* __restrict__ q_out, const T* __restrict__ qkv, long long ld, int lags,
                             const float* __restrict__ wt, float* __restrict__ state, const int* __restrict__ slot_ids,
                             const int* __restrict__ cu_seqlens, const int* __restrict__ context_lens,
                             const float* __restrict__ k_cs, int rot_dims, const float* __restrict__ v_cs,
                             const int* __restrict__ slot_mapping, T* __restrict__ k_pages, T* __restrict__ v_pages,
                             int page_size, int nq, int nkv, int dk, int dv, int dp) {
  constexpr int RUN = ONE ? 1 : TF_RUN;
  const int channels = (nq + nkv) * dk + nkv * dv;
  const int r = blockIdx.x, c = (blockIdx.y * 256 + threadIdx.x) * E;
  if (c >= channels) return;
  const int t0 = cu_seqlens[r], n = cu_seqlens[r + 1] - t0;
  int base = 0, seg = 1;
  if (!ONE) {
    const int lead = context_lens[r] & 7;          // the step's first position, relative to the multiple of 8 before it
    base = (blockIdx.z == 0 ? 0 : 8 + 8 * (int)blockIdx.z) - lead;
    seg = blockIdx.z == 0 ? 16 : 8;
  }
  const int i0 = max(0, base), i1 = min(n, base + seg);
  if (i0 >= i1) return;
  const int v_at = (nq + nkv) * dk;
  const bool is_v = c >= v_at, is_q = c < nq * dk;
  const int head = is_v ? (c - v_at) / dv : c / dk;                // k heads follow the q heads
  const int d0 = is_v ? (c - v_at) - head * dv : c - head * dk;
  const int kvh = is_v ? head : head - nq;
  float* st = state + (long long)slot_ids[r] * lags * channels + c;
  const T* in = qkv + (long long)t0 * ld + c;
  TfWindow<E, L> f;
  f.open(in, ld, i0, st, lags, channels, wt ? wt + c : nullptr);
  for (int b0 = base; b0 < i1; b0 += RUN) {
    typename TfVec<T, E>::type raw[RUN];
    int sm[RUN];
#pragma unroll
    for (int u = 0; u < RUN; ++u) {
      const int i = min(max(b0 + u, i0), i1 - 1);
      raw[u] = *(const typename TfVec<T, E>::type*)(in + (long long)i * ld);
      sm[u] = is_q ? -1 : slot_mapping[t0 + i];
    }
    TfPack8<T> pk[ONE ? 1 : E];
#pragma unroll
    for (int u = 0; u < RUN; ++u) {
      const int i = b0 + u;
      if (i < i0 || i >= i1) { sm[u] = -1; continue; }
      const long long t = t0 + i;
      float a[E], y[E];
      tf_widen<T, E>(raw[u], a);
      f.step(a, y);
      if (is_v) {
        if (v_cs) tf_turn<E>(y, v_cs + t * dv, dv >> 1, d0, dv);
        if constexpr (ONE) {
          if (sm[u] >= 0) {
            const long long page = sm[u] / page_size;
            T* dst = v_pages + ((page * nkv + kvh) * dp + d0) * (long long)page_size + (sm[u] - (int)page * page_size);
#pragma unroll
            for (int e = 0; e < E; ++e) dst[(long long)e * page_size] = from_f32<T>(y[e]);
          }
        } else {
#pragma unroll
          for (int e = 0; e < E; ++e) pk[e].v[u] = from_f32<T>(y[e]);
        }
        continue;
      }
      if (rot_dims) tf_turn<E>(y, k_cs + t * rot_dims, rot_dims >> 1, d0, rot_dims);
      if (is_q) {
        T* dst = q_out + (t * nq + head) * dp;
        tf_store<T, E>(dst + d0, y);
        if (d0 + E == dk)
          for (int p = dk; p < dp; ++p) dst[p] = from_f32<T>(0.f);
      } else if (sm[u] >= 0) {
        const long long page = sm[u] / page_size;
        tf_store<T, E>(k_pages + ((page * nkv + kvh) * page_size + (sm[u] - (int)page * page_size)) * (long long)dp + d0, y);
      }
    }
    if constexpr (!ONE) {
      if (!is_v) continue;
      bool side_by_side = sm[0] >= 0 && (sm[0] & 7) == 0 && (page_size & 7) == 0;      // 8 tokens at once
#pragma unroll
      for (int u = 1; u < RUN; ++u) side_by_side = side_by_side && sm[u] == sm[0] + u;
      if (side_by_side) {
        const long long page = sm[0] / page_size;
        T* dst = v_pages + ((page * nkv + kvh) * dp + d0) * (long long)page_size + (sm[0] - (int)page * page_size);
#pragma unroll
        for (int e = 0; e < E; ++e) *(TfPack8<T>*)(dst + (long long)e * page_size) = pk[e];
      } else {
#pragma unroll
        for (int u = 0; u < RUN; ++u) {
          if (sm[u] < 0) continue;
          const long long page = sm[u] / page_size;
          T* dst = v_pages + ((page * nkv + kvh) * dp + d0) * (long long)page_size + (sm[u] - (int)page * page_size);
#pragma unroll
          for (int e = 0; e < E; ++e) dst[(long long)e * page_size] = pk[e].v[u];
        }
      }
    }
  }
  if (blockIdx.z == 0 && lags > 0) tf_leave_state<T, E>(in, ld, n, st, lags, channels);
}

// ---------------------------------------------------------------- attention output
// o[t][h][0 .. dv) of rows [n][heads * dp], in place: the pairs (2m, 2m + 1) turn back by the token's angles v_cs
// [n][dv] (null: they stay), times sigmoid(g[t * ldg + h * dv + i]) (g null: no gate).
template <typename T, int E>
__global__ void __launch_bounds__(256)
rotate_back_gate_kernel(T* __restrict__ o, const T* __restrict__ g, long long ldg, const float* __restrict__ v_cs,
                        long long items, int heads, int dv, int dp) {
  const long long item = (long long)blockIdx.x * 256 + threadIdx.x;
  if (item >= items) return;
  const int per_head = dv / E, per_token = heads * per_head;
  const long long t = item / per_token;
  const int rest = (int)(item - t * per_token), h = rest / per_head, d0 = (rest - h * per_head) * E;
  T* dst = o + (t * heads + h) * (long long)dp + d0;
  float y[E];
  tf_load<T, E>(dst, y);
  if (v_cs) {
    const float* cs = v_cs + t * dv;
#pragma unroll
    for (int e = 0; e + 1 < E; e += 2) {
      const int m = (d0 + e) >> 1;
      const float c = cs[m], s = cs[(dv >> 1) + m];
      const float a = y[e], b = y[e + 1];
      y[e] = a * c + b * s;
      y[e + 1] = b * c - a * s;
    }
  }
  if (g) {
    float z[E];
    tf_load<T, E>(g + t * ldg + h * dv + d0, z);
#pragma unroll
    for (int e = 0; e < E; ++e) y[e] *= 1.f / (1.f + expf(-z[e]));
  }
  tf_store<T, E>(dst, y);
}

extern "C" int jv_token_filter_max_taps() { return TF_MAX_LAGS + 1; }

static bool tf_aligned(const void* p, size_t bytes) { return ((uintptr_t)p % bytes) == 0; }

template <typename T, int E>
static void launch_token_filter(dim3 grid, hipStream_t stream, T* out, const T* x, int channels, int lags, const float* wt,
                                float* state, const int* slot_ids, const int* cu_seqlens) {
  if (lags <= 3)
    hipLaunchKernelGGL((token_filter_kernel<T, E, 3>), grid, dim3(256), 0, stream, out, x, channels, lags, wt, state, slot_ids, cu_seqlens);
  else
    hipLaunchKernelGGL((token_filter_kernel<T, E, TF_MAX_LAGS>), grid, dim3(256), 0, stream, out, x, channels, lags, wt, state, slot_ids, cu_seqlens);
}

struct TfAttn {
  long long ld;
  int lags;
  const float* wt;
  float* state;
  const int *slot_ids, *cu_seqlens, *context_lens;
  const float* k_cs;
  int rot_dims;
  const float* v_cs;
  const int* slot_mapping;
  int page_size, nq, nkv, dk, dv, dp;
};

template <typename T, int E, int L>
static void launch_attn_prepare_filtered(dim3 grid, bool one, hipStream_t stream, T* q_out, const T* qkv, T* k_pages, T* v_pages, const TfAttn& a) {
  auto kernel = one ? attn_prepare_filtered_kernel<T, E, L, true> : attn_prepare_filtered_kernel<T, E, L, false>;
  hipLaunchKernelGGL(kernel, grid, dim3(256), 0, stream, q_out, qkv, a.ld, a.lags, a.wt, a.state,
                     a.slot_ids, a.cu_seqlens, a.context_lens, a.k_cs, a.rot_dims, a.v_cs, a.slot_mapping, k_pages, v_pages,
                     a.page_size, a.nq, a.nkv, a.dk, a.dv, a.dp);
}

#define DEFINE_TOKEN_FILTER(SUF, T)                                                                                \
  extern "C" int jv_token_filter_##SUF(void* out, const void* x, int channels, int taps, const float* wt,          \
                                       float* state, const int* slot_ids, const int* cu_seqlens, int n_requests,   \
                                       int max_q_len, void* stream) {                                              \
    if (n_requests <= 0 || channels <= 0 || max_q_len <= 0) return 0;                                              \
    if (taps < 1 || taps > TF_MAX_LAGS + 1 || !wt || (taps > 1 && !state)) return (int)hipErrorInvalidValue;                     \
    constexpr int EP = TF_BYTES / (int)sizeof(T);                                                                        \
    const bool vec = channels % EP == 0 && tf_aligned(out, 16) && tf_aligned(x, 16) && tf_aligned(wt, 32) &&       \
                     tf_aligned(state, 32);                                                                        \
    const int pieces = vec ? channels / EP : channels;                                                             \
    const int segs = (max_q_len + TF_RUN - 1) / TF_RUN;                                                            \
    if ((pieces + 255) / 256 > 65535 || segs > 65535) return (int)hipErrorInvalidValue;                            \
    const dim3 grid(n_requests, (pieces + 255) / 256, segs);                                                       \
    if (vec)                                                                                                       \
      launch_token_filter<T, EP>(grid, (hipStream_t)stream, (T*)out, (const T*)x, channels, taps - 1, wt, state, slot_ids, cu_seqlens); \
    else                                                                                                           \
      launch_token_filter<T, 1>(grid, (hipStream_t)stream, (T*)out, (const T*)x, channels, taps - 1, wt, state, slot_ids, cu_seqlens); \
    return JV_LAUNCH_CHECK();                                                                                      \
  }                                                                                                                \
  extern "C" int jv_attn_prepare_filtered_##SUF(                                                                   \
      void* q_out, const void* qkv, long long ld, int taps, const float* wt, float* state, const int* slot_ids,    \
      const int* cu_seqlens, const int* context_lens, const float* k_cs, int rot_dims, const float* v_cs,          \
      const int* slot_mapping, void* k_pages, void* v_pages, int page_size, int n_requests, int max_q_len, int nq, \
      int nkv, int dk, int dv, int dp, void* stream) {                                                             \
    if (n_requests <= 0 || max_q_len <= 0) return 0;                                                               \
    if (taps < 1 || taps > TF_MAX_LAGS + 1 || (taps > 1 && (!wt || !state || !slot_ids)) || nq <= 0 || nkv <= 0 || \
        !slot_ids || dk <= 0 || dv <= 0 || dk % 2 || dv % 2 || dp < dk || dp < dv || rot_dims < 0 || rot_dims > dk ||           \
        rot_dims % 2 || (rot_dims && !k_cs) || !slot_mapping || !k_pages || !v_pages || page_size <= 0)            \
      return (int)hipErrorInvalidValue;                                                                            \
    constexpr int EP = TF_BYTES / (int)sizeof(T);                                                                        \
    const bool vec = dk % EP == 0 && dv % EP == 0 && dp % EP == 0 && ld % EP == 0 && tf_aligned(qkv, 16) &&        \
                     tf_aligned(q_out, 16) && tf_aligned(k_pages, 16) && tf_aligned(wt, 32) && tf_aligned(state, 32); \
    if (!vec && (dp % 2 || ld % 2)) return (int)hipErrorInvalidValue;                                              \
    if (page_size % 8 == 0 && !tf_aligned(v_pages, 8 * sizeof(T))) return (int)hipErrorInvalidValue;               \
    const int channels = (nq + nkv) * dk + nkv * dv, pieces = channels / (vec ? EP : 2);                           \
    const int segs = max_q_len <= 9 ? 1 : (max_q_len + 7 - 16 + 7) / 8 + 1;                                        \
    if ((pieces + 255) / 256 > 65535 || segs > 65535) return (int)hipErrorInvalidValue;                            \
    const TfAttn a{ld, taps - 1, wt, state, slot_ids, cu_seqlens, context_lens, k_cs, rot_dims, v_cs, slot_mapping, \
                   page_size, nq, nkv, dk, dv, dp};                                                                \
    const dim3 grid(n_requests, (pieces + 255) / 256, segs);                                                       \
    auto launch = vec ? (taps <= 4 ? launch_attn_prepare_filtered<T, EP, 3>                                        \
                                   : launch_attn_prepare_filtered<T, EP, TF_MAX_LAGS>)                             \
                      : (taps <= 4 ? launch_attn_prepare_filtered<T, 2, 3>                                         \
                                   : launch_attn_prepare_filtered<T, 2, TF_MAX_LAGS>);                             \
    launch(grid, max_q_len == 1, (hipStream_t)stream, (T*)q_out, (const T*)qkv, (T*)k_pages, (T*)v_pages, a);                      \
    return JV_LAUNCH_CHECK();                                                                                      \
  }                                                                                                                \
  extern "C" int jv_rotate_back_gate_##SUF(void* o, const void* g, long long ldg, const float* v_cs, long long n,  \
                                           int heads, int dv, int dp, void* stream) {                              \
    if (n <= 0 || heads <= 0) return 0;                                                                            \
    if (dv <= 0 || dp < dv || (v_cs && dv % 2)) return (int)hipErrorInvalidValue;                                  \
    constexpr int EP = TF_BYTES / (int)sizeof(T);                                                                        \
    const bool vec = dv % EP == 0 && dp % EP == 0 && tf_aligned(o, 16) && (!g || (ldg % EP == 0 && tf_aligned(g, 16))); \
    const bool two = dv % 2 == 0 && dp % 2 == 0 && (!g || (ldg % 2 == 0 && tf_aligned(g, 2 * sizeof(T))));         \
    if (!vec && !two && v_cs) return (int)hipErrorInvalidValue;                                                    \
    const long long items = n * heads * (dv / (vec ? EP : two ? 2 : 1));                                           \
    if ((items + 255) / 256 > 0x7fffffffll) return (int)hipErrorInvalidValue;                                      \
    const dim3 grid((unsigned)((items + 255) / 256));                                                              \
    if (vec)                                                                                                       \
      hipLaunchKernelGGL((rotate_back_gate_kernel<T, EP>), grid, dim3(256), 0, (hipStream_t)stream, (T*)o,         \
                         (const T*)g, ldg, v_cs, items, heads, dv, dp);                                            \
    else if (two)                                                                                                  \
      hipLaunchKernelGGL((rotate_back_gate_kernel<T, 2>), grid, dim3(256), 0, (hipStream_t)stream, (T*)o,          \
                         (const T*)g, ldg, v_cs, items, heads, dv, dp);                                            \
    else                                                                                                           \
      hipLaunchKernelGGL((rotate_back_gate_kernel<T, 1>), grid, dim3(256), 0, (hipStream_t)stream, (T*)o,          \
                         (const T*)g, ldg, v_cs, items, heads, dv, dp);                                            \
    return JV_LAUNCH_CHECK();                                                                                      \
  }

DEFINE_TOKEN_FILTER(bf16, bf16_t)
DEFINE_TOKEN_FILTER(f32, float)
