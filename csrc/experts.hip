// Mixture of gated experts with an optional shared expert (gfx950).
//
//   route   router logits -> chosen experts and their weights: the softmax
//           over the chosen, or with a correction the softmax over all, the
//           correction added for the choice only; sigmoid of the shared
//           expert's gate.  Outputs after the E experts are identity experts
//           (choice -1)
//   sort    choices by expert, in tiles of `bm` rows; for few tokens routing
//           and sorting are one kernel.  The shared expert may be expert
//           number E, chosen by every token
//   up      h = silu(x W_gate) * (x W_up) of every choice, or the clamped
//           g sigmoid(1.702 g) (u + 1)
//   down    y = h W_down of every choice
//   sum     weighted sum of a token's choices, and either the sum itself or
//           its RMS norm added to the float residual; or the whole step to
//           the next sublayer's input (sublayer.h)
//
// Every grid depends on shapes only.  up and down stream each expert's
// weights once per tile: weights are the A operand straight from memory, the
// tile's rows the B operand, and the four waves of a workgroup divide K.  The
// general kernels take any sizes, bf16 or float, with bm = 1.
#include <float.h>

#include <algorithm>

#include "sublayer.h"

namespace {

constexpr int ROUTE_TOGETHER = 64;   // tokens routed by the sorting workgroup

struct Route {
  float* weight;           // [T, n]
  int* ids;                // [T, n] or null
  const float* logits;     // [T, N (+ 1)], N = E + identity
  int T, E, top, shared;   // n = top + shared where ids has the shared expert
  int with_shared;         // ids lists the shared expert
  int N;
  const float* correction; // [N] or null
};

// One wave: the `top` <= 64 largest of N <= 64 * LE logits (or corrected
// shares) by repeated maximum, lowest index first among equals; a logit that
// is not a number ranks last.  Lane k returns choice k (-1: an identity
// expert) and its weight.
template <int LE>
DEV void route_token(const Route& r, const float* z, int* id, float* weight) {
  const int lane = threadIdx.x & 63, E = r.N, top = r.top;
  float v[LE], share[LE];
  #pragma unroll
  for (int i = 0; i < LE; ++i)       // the maximum drops NaN
    v[i] = lane + 64 * i < E ? fmaxf(z[lane + 64 * i], -FLT_MAX) : 0.f;
  if (r.correction) {
    float mx = -FLT_MAX, sum = 0.f;
    #pragma unroll
    for (int i = 0; i < LE; ++i)
      if (lane + 64 * i < E) mx = fmaxf(mx, v[i]);
    mx = wave_reduce_max(mx);
    #pragma unroll
    for (int i = 0; i < LE; ++i) {
      share[i] = lane + 64 * i < E ? expf(v[i] - mx) : 0.f;
      sum += share[i];
    }
    sum = wave_reduce_sum(sum);
    #pragma unroll
    for (int i = 0; i < LE; ++i) {
      share[i] /= sum;
      if (lane + 64 * i < E) v[i] = share[i] + r.correction[lane + 64 * i];
    }
  }
  unsigned taken = 0;
  float first = 0.f;
  *id = -1;
  *weight = 0.f;
  for (int k = 0; k < top; ++k) {
    float best = -INFINITY;
    int at = INT_MAX;
    #pragma unroll
    for (int i = 0; i < LE; ++i)
      if (lane + 64 * i < E && !(taken >> i & 1) &&
          (at == INT_MAX || v[i] > best)) {
        best = v[i];
        at = lane + 64 * i;
      }
    #pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float b = __shfl_xor(best, o);
      const int a = __shfl_xor(at, o);
      if (a != INT_MAX &&
          (at == INT_MAX || b > best || (b == best && a < at))) {
        best = b;
        at = a;
      }
    }
    if ((at & 63) == lane) taken |= 1u << (at >> 6);
    if (k == 0) first = best;
    float s = 0.f;
    if (r.correction) {
      #pragma unroll
      for (int i = 0; i < LE; ++i)
        if (at >> 6 == i) s = share[i];
      s = __shfl(s, at & 63);
    }
    if (lane == k) {
      *id = at < r.E ? at : -1;
      *weight = r.correction ? s : expf(best - first);
    }
  }
  if (!r.correction) *weight /= wave_reduce_sum(*weight);
  if (r.shared && lane == top) {
    *id = r.E;
    *weight = 1.f / (1.f + expf(-z[E]));
  }
}

template <int LE>
DEV void route_row(const Route& r, int t) {
  const int lane = threadIdx.x & 63, n = r.top + r.shared;
  int id;
  float w;
  route_token<LE>(r, r.logits + (long)t * (r.N + r.shared), &id, &w);
  if (lane < n) r.weight[(long)t * n + lane] = w;
  const int m = r.top + r.with_shared;
  if (lane < m) r.ids[(long)t * m + lane] = id;
}

template <int LE>
__global__ __launch_bounds__(256) void route_kernel(Route r) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t < r.T) route_row<LE>(r, t);
}

// One workgroup.  order[pos] = choice (-1: padding), expert[tile] (-1: none),
// place[choice] = pos (-1: an identity expert).  ROUTE: the choices are made
// here first.
template <int LE, bool ROUTE>
__global__ __launch_bounds__(1024) void sort_kernel(
    Route r, int* __restrict__ order, int* __restrict__ expert,
    int* __restrict__ place, const int* ids, int choices, int kinds, int bm,
    int tiles) {
  extern __shared__ int lds[];
  int* cnt = lds;                    // choices per expert
  int* cur = lds + kinds;            // next free position
  __shared__ int wave_sum[16];
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  for (int e = tid; e < kinds; e += 1024) cnt[e] = 0;
  for (int i = tid; i < tiles * bm; i += 1024) order[i] = -1;
  for (int t = tid; t < tiles; t += 1024) expert[t] = -1;
  if constexpr (ROUTE)
    for (int t = wid; t < r.T; t += 16) route_row<LE>(r, t);
  __threadfence_block();
  __syncthreads();
  for (int p = tid; p < choices; p += 1024)
    if (ids[p] >= 0) atomicAdd(&cnt[ids[p]], 1);
  __syncthreads();
  // exclusive sums of tiles: kinds <= 1024 + 1, one or two a thread
  int base = 0;
  for (int e0 = 0; e0 < kinds; e0 += 1024) {
    const int e = e0 + tid;
    const int n = e < kinds ? (cnt[e] + bm - 1) / bm : 0;
    int x = n;
    #pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int v = __shfl_up(x, o);
      if (lane >= o) x += v;
    }
    if (lane == 63) wave_sum[wid] = x;
    __syncthreads();
    int before = base, total = base;
    for (int w = 0; w < 16; ++w) {
      if (w < wid) before += wave_sum[w];
      total += wave_sum[w];
    }
    const int first = before + x - n;
    if (e < kinds) {
      cur[e] = first * bm;
      for (int t = first; t < first + n && t < tiles; ++t) expert[t] = e;
    }
    base = total;
    __syncthreads();
  }
  for (int p = tid; p < choices; p += 1024) {
    const int pos = ids[p] < 0 ? -1 : atomicAdd(&cur[ids[p]], 1);
    if (pos >= 0) order[pos] = p;
    place[p] = pos;
  }
}

// ---- products -------------------------------------------------------------
// UP:   out[p, f] = act(x . w[e, f], x . w[e, N + f]), x row order[p]/div
// else: out[p, n] = x . w[e, n], x row p
// w [E, UP ? 2N : N, K]; the shared expert (e == E) has ws, Ns, Ks.
struct Grouped {
  const int* order;
  const int* expert;
  int E, N, K, Ns, Ks, div;
  long xs, os;                       // row strides of x and out
  int clamped;
  float limit;
};

template <typename T> DEV float gate_act(const Grouped& a, float g, float u) {
  return a.clamped ? clamped_unit<T>(g, u, a.limit)
                   : g / (1.f + Fn<T>::exp(-g)) * u;
}

template <int CT, int NA, bool UP>
__global__ __launch_bounds__(256) void experts_rows_kernel(
    bf16* __restrict__ out, const bf16* __restrict__ x,
    const bf16* __restrict__ w, const bf16* __restrict__ ws, Grouped a) {
  constexpr int BM = 16 * CT, COLS = UP ? NA * 8 : NA * 16;
  extern __shared__ __attribute__((aligned(16))) float red[];
  const int tile = blockIdx.y, e = a.expert[tile];
  if (e < 0) return;
  const bool shared = e == a.E;
  const int N = shared ? a.Ns : a.N, K = shared ? a.Ks : a.K;
  const int n0 = blockIdx.x * COLS;
  if (n0 >= N) return;
  const bf16* we = shared ? ws : w + (long)e * (UP ? 2 * N : N) * K;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int col = lane & 15, gr = lane >> 4;

  const bf16* wp[NA];
  bool wl[NA];
  #pragma unroll
  for (int i = 0; i < NA; ++i) {
    const int half = UP ? i / (NA / 2) : 0, j = UP ? i % (NA / 2) : i;
    const int n = n0 + j * 16 + col;
    wl[i] = n < N;
    wp[i] = we + ((long)half * N + (wl[i] ? n : 0)) * K + gr * 8;
  }
  const bf16* xp[CT];
  bool xl[CT];
  #pragma unroll
  for (int t = 0; t < CT; ++t) {
    const int p = tile * BM + t * 16 + col;
    const int choice = a.order[p];
    xl[t] = choice >= 0;
    xp[t] = x + (UP ? (xl[t] ? choice / a.div : 0) : p) * a.xs + gr * 8;
  }
  f32x4_t acc[NA][CT];
  #pragma unroll
  for (int i = 0; i < NA; ++i)
    #pragma unroll
    for (int t = 0; t < CT; ++t) acc[i][t] = f32x4_t(0.f);
  #pragma unroll 2
  for (int k0 = wid * 64; k0 < K; k0 += 256) {
    short8_t wf[2][NA], xf[2][CT];
    #pragma unroll
    for (int s = 0; s < 2; ++s) {
      const int k = k0 + 32 * s;
      const bool in = k + gr * 8 < K;
      #pragma unroll
      for (int i = 0; i < NA; ++i)
        wf[s][i] = in && wl[i]
            ? *reinterpret_cast<const short8_t*>(wp[i] + k) : short8_t{};
      #pragma unroll
      for (int t = 0; t < CT; ++t)
        xf[s][t] = in && xl[t]
            ? *reinterpret_cast<const short8_t*>(xp[t] + k) : short8_t{};
    }
    #pragma unroll
    for (int s = 0; s < 2; ++s)
      #pragma unroll
      for (int i = 0; i < NA; ++i)
        #pragma unroll
        for (int t = 0; t < CT; ++t)
          acc[i][t] = mfma16(wf[s][i], xf[s][t], acc[i][t]);
  }
  #pragma unroll
  for (int i = 0; i < NA; ++i)
    #pragma unroll
    for (int t = 0; t < CT; ++t)
      *reinterpret_cast<f32x4_t*>(
          red + (((wid * NA + i) * CT + t) * 64 + lane) * 4) = acc[i][t];
  __syncthreads();
  auto total = [&](int i, int t) {
    f32x4_t s = f32x4_t(0.f);
    #pragma unroll
    for (int v = 0; v < 4; ++v)
      s += *reinterpret_cast<const f32x4_t*>(
          red + (((v * NA + i) * CT + t) * 64 + lane) * 4);
    return s;
  };
  constexpr int NI = UP ? NA / 2 : NA;
  for (int u = wid; u < NI * CT; u += 4) {
    const int i = u / CT, t = u % CT;
    const int n = n0 + i * 16 + gr * 4;
    const long p = tile * BM + t * 16 + col;
    if (n >= N || a.order[p] < 0) continue;   // N is a multiple of 8
    f32x4_t y = total(i, t);
    if constexpr (UP) {
      const f32x4_t z = total(i + NA / 2, t);
      #pragma unroll
      for (int j = 0; j < 4; ++j) y[j] = gate_act<bf16>(a, y[j], z[j]);
    }
    *reinterpret_cast<uint2*>(out + p * a.os + n) =
        uint2{cvt_pk_bf16(y[0], y[1]), cvt_pk_bf16(y[2], y[3])};
  }
}

// bm = 1: row p alone; a wave has 16 n
template <typename T, bool UP>
__global__ __launch_bounds__(256) void experts_general_kernel(
    T* __restrict__ out, const T* __restrict__ x, const T* __restrict__ w,
    const T* __restrict__ ws, Grouped a) {
  const int p = blockIdx.x, e = a.expert[p];
  if (e < 0) return;
  const bool shared = e == a.E;
  const int N = shared ? a.Ns : a.N, K = shared ? a.Ks : a.K;
  const T* we = shared ? ws : w + (long)e * (UP ? 2 * N : N) * K;
  const T* xp = x + (UP ? a.order[p] / a.div : p) * a.xs;
  const int lane = threadIdx.x & 63;
  const int n0 = (blockIdx.y * 4 + (threadIdx.x >> 6)) * 16;
  for (int n = n0; n < min(n0 + 16, N); ++n) {
    float s = 0.f, z = 0.f;
    for (int k = lane; k < K; k += 64) {
      const float xv = Elem<T>::ld(xp + k);
      s += xv * Elem<T>::ld(we + (long)n * K + k);
      if constexpr (UP) z += xv * Elem<T>::ld(we + (long)(N + n) * K + k);
    }
    s = wave_reduce_sum(s);
    if constexpr (UP) {
      z = wave_reduce_sum(z);
      s = gate_act<T>(a, s, z);
    }
    if (lane == 0) Elem<T>::st(out + p * a.os + n, s);
  }
}

// ---- weighted sum, norm, residual -----------------------------------------
// h[t] = sum_k weight[t, k] y[place[t, k]]  (+ weight[t, n] shared[t]), with
// identity[t] where place is -1 (null: that part is added elsewhere)
template <typename T> struct Sum {
  const T* y;
  const T* shared;
  const T* identity;
  const float* weight;
  const int* place;
  int n, width;

  template <int V> DEV void value(long t, int c, float* h) const {
    const int nw = n + (shared ? 1 : 0);
    #pragma unroll
    for (int i = 0; i < V; ++i) h[i] = 0.f;
    for (int k = 0; k < nw; ++k) {
      const T* row = shared + t * width;
      if (k < n) {
        const int p = place[t * n + k];
        if (p < 0 && !identity) continue;
        row = p < 0 ? identity + t * width : y + (long)p * width;
      }
      const float wk = weight[t * nw + k];
      float f[V];
      load_vec<T, V>(row + c, f);
      #pragma unroll
      for (int i = 0; i < V; ++i) h[i] += wk * f[i];
    }
  }
};

// without a residual out = h, otherwise residual += rms(h) * w and out = the
// residual (null: none).  One workgroup a token.
template <typename T, int V>
__global__ __launch_bounds__(256) void experts_sum_kernel(
    T* __restrict__ out, float* __restrict__ residual, Sum<T> s,
    const float* __restrict__ w, float eps) {
  constexpr int HELD = 4;
  __shared__ float scratch[4];
  const int tid = threadIdx.x, width = s.width;
  const long t = blockIdx.x, at = t * width;
  auto value = [&](int c, float* h) { s.template value<V>(t, c, h); };
  if (!residual) {
    for (int c = tid * V; c < width; c += 256 * V) {
      float h[V];
      value(c, h);
      store_vec<T, V>(out + at + c, h);
    }
    return;
  }
  float held[HELD][V], ss = 0.f;
  #pragma unroll
  for (int i = 0; i < HELD; ++i) {
    const int c = (i * 256 + tid) * V;
    if (c < width) {
      value(c, held[i]);
      #pragma unroll
      for (int j = 0; j < V; ++j) ss += held[i][j] * held[i][j];
    }
  }
  for (int c = (HELD * 256 + tid) * V; c < width; c += 256 * V) {
    float h[V];
    value(c, h);
    #pragma unroll
    for (int j = 0; j < V; ++j) ss += h[j] * h[j];
  }
  ss = block_reduce_sum_256(ss, scratch);
  const float rs = 1.f / sqrtf(ss / width + eps);
  auto add = [&](int c, const float* h) {
    float wv[V], r[V];
    load_vec<float, V>(w + c, wv);
    load_vec<float, V>(residual + at + c, r);
    #pragma unroll
    for (int j = 0; j < V; ++j) r[j] += h[j] * rs * wv[j];
    store_vec<float, V>(residual + at + c, r);
    if (out) store_vec<T, V>(out + at + c, r);
  };
  #pragma unroll
  for (int i = 0; i < HELD; ++i) {
    const int c = (i * 256 + tid) * V;
    if (c < width) add(c, held[i]);
  }
  for (int c = (HELD * 256 + tid) * V; c < width; c += 256 * V) {
    float h[V];
    value(c, h);
    add(c, h);
  }
}

template <typename T, int V, int NT, bool CONV>
__global__ __launch_bounds__(NT) void experts_sum_next_kernel(Between<T> a,
                                                              Sum<T> s) {
  const long t = blockIdx.x;
  between_sublayers<T, V, NT, CONV, ADD_NORMED>(a, t, [&](int c, float* x) {
    s.template value<V>(t, c, x);
  });
}

}  // namespace

#define BY_EXPERTS(RUN)                                                     \
  if (r.N <= 64) RUN(1);                                                    \
  else if (r.N <= 256) RUN(4);                                              \
  else RUN(16)

// ids lists [T, top] or, with_shared, [T, top + 1]; at most 1024 outputs,
// top <= 63
void launch_experts_route(float* weight, int* ids, const float* logits, int T,
                          int E, int top, bool shared, bool with_shared,
                          int identity, const float* correction,
                          hipStream_t stream) {
  if (T == 0) return;
  const Route r{weight, ids, logits, T, E, top, shared, with_shared,
                E + identity, correction};
  #define RUN(LE)                                                           \
    route_kernel<LE><<<(unsigned)((T + 3) / 4), 256, 0, stream>>>(r)
  BY_EXPERTS(RUN);
  #undef RUN
}

void launch_experts_sort(int* order, int* expert, int* place, const int* ids,
                         int choices, int kinds, int bm, int tiles,
                         hipStream_t stream) {
  sort_kernel<1, false><<<1, 1024, 2 * kinds * sizeof(int), stream>>>(
      Route{}, order, expert, place, ids, choices, kinds, bm, tiles);
}

void launch_experts_route_sort(float* weight, int* ids, int* place,
                               int* order, int* expert, const float* logits,
                               int T, int E, int top, bool shared, int bm,
                               int tiles, int identity,
                               const float* correction, hipStream_t stream) {
  if (T == 0) return;
  const int kinds = E + shared, choices = T * (top + shared);
  if (T > ROUTE_TOGETHER) {
    launch_experts_route(weight, ids, logits, T, E, top, shared, shared,
                         identity, correction, stream);
    launch_experts_sort(order, expert, place, ids, choices, kinds, bm, tiles,
                        stream);
    return;
  }
  const Route r{weight, ids, logits, T, E, top, shared, shared, E + identity,
                correction};
  #define RUN(LE)                                                           \
    sort_kernel<LE, true><<<1, 1024, 2 * kinds * sizeof(int), stream>>>(    \
        r, order, expert, place, ids, choices, kinds, bm, tiles)
  BY_EXPERTS(RUN);
  #undef RUN
}

// bm 16, 32 or 64: matrix cores (bf16, N and K multiples of 8); bm 1: general
template <typename T>
void launch_experts_gemm(bool up, T* out, const T* x, const T* w, const T* ws,
                         const int* order, const int* expert, int tiles,
                         int E, int N, int K, int Ns, int Ks, int div,
                         long xs, long os, int bm, bool clamped, float limit,
                        hipStream_t stream) {
  if (tiles == 0) return;
  const Grouped a{order, expert, E, N, K, Ns, Ks, div, xs, os, clamped, limit};
  const int n = std::max(N, Ns);
  if (bm == 1) {
    const dim3 grid((unsigned)tiles, (unsigned)((n + 63) / 64));
    if (up)
      experts_general_kernel<T, true><<<grid, 256, 0, stream>>>(out, x, w, ws,
                                                                a);
    else
      experts_general_kernel<T, false><<<grid, 256, 0, stream>>>(out, x, w,
                                                                 ws, a);
    return;
  }
  if constexpr (sizeof(T) == 2) {
    #define RUN(CT, NA, UP)                                                 \
      {                                                                     \
        const int cols = UP ? NA * 8 : NA * 16, lds = NA * CT * 4096;       \
        experts_rows_kernel<CT, NA, UP>                                     \
            <<<dim3((unsigned)((n + cols - 1) / cols), (unsigned)tiles),    \
               256, lds, stream>>>(out, x, w, ws, a);                       \
      }
    #define BY_ROWS(UP)                                                     \
      if (bm == 16) RUN(1, 2, UP)                                           \
      else if (bm == 32) RUN(2, 4, UP)                                      \
      else RUN(4, 4, UP)
    if (up) {
      BY_ROWS(true)
    } else {
      BY_ROWS(false)
    }
    #undef BY_ROWS
    #undef RUN
  }
}

template <typename T>
void launch_experts_sum(T* out, float* residual, const T* y, const T* shared,
                        const T* identity, const float* weight,
                        const int* place, const float* w, long rows, int n,
                        int width, float eps, hipStream_t stream) {
  if (rows == 0) return;
  const Sum<T> s{y, shared, identity, weight, place, n, width};
  if (width % 4 == 0)
    experts_sum_kernel<T, 4><<<(unsigned)rows, 256, 0, stream>>>(
        out, residual, s, w, eps);
  else
    experts_sum_kernel<T, 1><<<(unsigned)rows, 256, 0, stream>>>(
        out, residual, s, w, eps);
}

template <typename T>
void launch_experts_sum_next(const Between<T>& a, const T* y, const T* shared,
                             const T* identity, const float* weight,
                             const int* place, long rows, int n,
                             hipStream_t stream) {
  if (rows == 0) return;
  const Sum<T> s{y, shared, identity, weight, place, n, a.width};
  #define RUN(V, NT, CONV)                                                  \
    experts_sum_next_kernel<T, V, NT, CONV>                                 \
        <<<(unsigned)rows, NT, 0, stream>>>(a, s)
  BY_WIDTH(RUN);
  #undef RUN
}

#define INSTANTIATE(T)                                                      \
  template void launch_experts_gemm<T>(                                     \
      bool, T*, const T*, const T*, const T*, const int*, const int*, int,  \
      int, int, int, int, int, int, long, long, int, bool, float,           \
      hipStream_t);                                                         \
  template void launch_experts_sum<T>(                                      \
      T*, float*, const T*, const T*, const T*, const float*, const int*,   \
      const float*, long, int, int, float, hipStream_t);                    \
  template void launch_experts_sum_next<T>(                                 \
      const Between<T>&, const T*, const T*, const T*, const float*,        \
      const int*, long, int, hipStream_t);
INSTANTIATE(bf16)
INSTANTIATE(float)
#undef INSTANTIATE
