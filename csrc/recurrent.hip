// Linear recurrences with a matrix state per head (gfx950): gated linear
// attention (decay per key channel), the matrix-memory LSTM (scalar
// exponential gates with a running maximum) and lightning attention (a
// constant decay per head, SiLU on q, k and v, norm over all heads outside).
//
//   S_t = diag(a_t) S_{t-1} + k_t v_t^T          o_t = S_t^T q_t
//
// State pool, float, indexed by the sequence's state slot:
//   S [slots, H, D, E]   and for the matrix LSTM  n [slots, H, D], m [slots, H]
// A sequence's first token (position 0) starts from zero whatever the slot
// holds, so slots need no clearing between sequences.
//
// This file holds the decode step (one token per sequence, output
// normalisation and gate fused), the token-by-token scan that serves any size
// and element type, and the elementwise pieces around the scan.
#include "common.h"
#include "recurrent.h"

namespace {

// what enters the recurrence from a projection
template <typename T, Kind K> DEV float entry(const T* p) {
  const float x = Elem<T>::ld(p);
  if constexpr (K == LIGHTNING) return x / (1.f + Fn<T>::exp(-x));
  return x;
}

// z = a2[row] . a1h + b ; log decay = log_sigmoid(z) / tau
template <typename T>
DEV float gla_log_decay(const T* a1h, const T* a2, const float* b, int c,
                        int rank, float inv_tau) {
  float z = b[c];
  for (int r = 0; r < rank; ++r)
    z += Elem<T>::ld(a1h + r) * Elem<T>::ld(a2 + (long)c * rank + r);
  return log_sigmoid(z) * inv_tau;
}

DEV void mlstm_gates(float zi, float zf, float cap, float* i, float* f) {
  *i = cap * tanhf(zi / cap);
  *f = log_sigmoid(cap * tanhf(zf / cap));
}

template <typename T>
__global__ __launch_bounds__(256) void gla_decay_kernel(
    float* __restrict__ log_decay, const T* __restrict__ a1h,
    const T* __restrict__ a2, const float* __restrict__ a2b, int channels,
    int rank, float inv_tau, long stride) {
  const long t = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c < channels)
    log_decay[t * channels + c] =
        gla_log_decay<T>(a1h + t * stride, a2, a2b, c, rank, inv_tau);
}

// gates [T, 2H] raw (input | forget) -> log gates in place of the same layout
__global__ __launch_bounds__(256) void mlstm_gates_kernel(
    float* __restrict__ out, const float* __restrict__ raw,
    const float* __restrict__ ib, const float* __restrict__ fb, long rows,
    int H, float cap) {
  const long u = (long)blockIdx.x * 256 + threadIdx.x;
  if (u >= rows * H) return;
  const long t = u / H;
  const int h = (int)(u % H);
  float i, f;
  mlstm_gates(raw[t * 2 * H + h] + ib[h], raw[t * 2 * H + H + h] + fb[h],
              cap, &i, &f);
  out[t * 2 * H + h] = i;
  out[t * 2 * H + H + h] = f;
}

// ---- token scan ----------------------------------------------------------
// One wave owns COLS columns of one head's state for one sequence; a lane
// holds RPL rows of them.  o is written unnormalised, float [T, H, E].
constexpr int COLS = 4;

template <typename T, int RPL, Kind K>
__global__ __launch_bounds__(64) void recurrent_scan_kernel(
    float* __restrict__ o, float* __restrict__ S,
    const float* __restrict__ n_pool, const float* __restrict__ m_pool,
    float* __restrict__ nm_new, const T* __restrict__ q,
    const T* __restrict__ k, const T* __restrict__ v,
    const float* __restrict__ gates, const int* __restrict__ seq_start,
    const long* __restrict__ positions, const int* __restrict__ slots,
    int H, int D, int E, long stride, float qscale) {
  const int lane = threadIdx.x;
  const int e0 = blockIdx.x * COLS;
  const int h = blockIdx.y;
  const int s = blockIdx.z;
  const int t0 = seq_start[s], t1 = seq_start[s + 1];
  const int slot = slots[s];
  if (t0 >= t1) return;
  const bool fresh = positions[t0] == 0 || slot < 0;
  float st[RPL][COLS], nv[RPL], m = 0.f;
  float* Sp = S + ((long)max(slot, 0) * H + h) * D * E;
  #pragma unroll
  for (int r = 0; r < RPL; ++r) {
    const int d = lane + 64 * r;
    nv[r] = 0.f;
    if (K == MLSTM && !fresh && d < D)
      nv[r] = n_pool[((long)slot * H + h) * D + d];
    #pragma unroll
    for (int c = 0; c < COLS; ++c)
      st[r][c] = (!fresh && d < D && e0 + c < E)
          ? Sp[(long)d * E + e0 + c] : 0.f;
  }
  if (K == MLSTM && !fresh) m = m_pool[(long)slot * H + h];

  for (int t = t0; t < t1; ++t) {
    float fs = K == LIGHTNING ? gates[h] : 1.f, is = 1.f;
    if constexpr (K == MLSTM) {
      const float li = gates[(long)t * 2 * H + h];
      const float lf = gates[(long)t * 2 * H + H + h];
      const float mn = fmaxf(lf + m, li);
      fs = expf(lf + m - mn);
      is = expf(li - mn);
      m = mn;
    }
    float vv[COLS], acc[COLS], den = 0.f;
    #pragma unroll
    for (int c = 0; c < COLS; ++c) {
      vv[c] = e0 + c < E
          ? entry<T, K>(v + (long)t * stride + (long)h * E + e0 + c) : 0.f;
      acc[c] = 0.f;
    }
    #pragma unroll
    for (int r = 0; r < RPL; ++r) {
      const int d = lane + 64 * r;
      const bool in = d < D;
      const long at = (long)t * stride + (long)h * D + d;
      const float qd = in ? entry<T, K>(q + at) * qscale : 0.f;
      const float kd = in ? entry<T, K>(k + at) * is : 0.f;
      float a = fs;
      if constexpr (K == GLA)
        a = in ? expf(gates[((long)t * H + h) * D + d]) : 0.f;
      if constexpr (K == MLSTM) {
        nv[r] = nv[r] * a + kd;
        den += nv[r] * qd;
      }
      #pragma unroll
      for (int c = 0; c < COLS; ++c) {
        st[r][c] = st[r][c] * a + kd * vv[c];
        acc[c] += st[r][c] * qd;
      }
    }
    #pragma unroll
    for (int c = 0; c < COLS; ++c) acc[c] = wave_reduce_sum(acc[c]);
    float inv = 1.f;
    if constexpr (K == MLSTM) {
      den = wave_reduce_sum(den);
      inv = 1.f / (fmaxf(fabsf(den), expf(-m)) + DEN_EPS);
    }
    if (lane == 0) {
      #pragma unroll
      for (int c = 0; c < COLS; ++c)
        if (e0 + c < E)
          o[((long)t * H + h) * E + e0 + c] = acc[c] * inv;
    }
  }
  if (slot < 0) return;
  #pragma unroll
  for (int r = 0; r < RPL; ++r) {
    const int d = lane + 64 * r;
    if (d >= D) continue;
    #pragma unroll
    for (int c = 0; c < COLS; ++c)
      if (e0 + c < E) Sp[(long)d * E + e0 + c] = st[r][c];
    // every column block carries the same n and m; the first one hands them
    // on (not into the pool: other column blocks may still read it)
    if (K == MLSTM && e0 == 0) nm_new[((long)s * H + h) * (D + 1) + d] = nv[r];
  }
  if (K == MLSTM && e0 == 0 && lane == 0)
    nm_new[((long)s * H + h) * (D + 1) + D] = m;
}

// n and m of every sequence from a finished prefill into the pool
__global__ __launch_bounds__(256) void mlstm_commit_kernel(
    float* __restrict__ n_pool, float* __restrict__ m_pool,
    const float* __restrict__ nm_new, const int* __restrict__ seq_start,
    const int* __restrict__ slots, int H, int D) {
  const int h = blockIdx.x, s = blockIdx.y;
  const int slot = slots[s];
  if (slot < 0 || seq_start[s] >= seq_start[s + 1]) return;
  const float* src = nm_new + ((long)s * H + h) * (D + 1);
  for (int d = threadIdx.x; d < D; d += 256)
    n_pool[((long)slot * H + h) * D + d] = src[d];
  if (threadIdx.x == 0) m_pool[(long)slot * H + h] = src[D];
}

// ---- output: per-head RMS norm, weight, gate ------------------------------
template <typename T, Kind K>
DEV float out_gate(float g) {
  const float sg = 1.f / (1.f + Fn<T>::exp(-g));
  return K == MLSTM ? sg : g * sg;
}

// one workgroup per (token, head): y = rms(o) * w * gate(g)
template <typename T, Kind K>
__global__ __launch_bounds__(256) void recurrent_out_kernel(
    T* __restrict__ y, const float* __restrict__ o, const T* __restrict__ g,
    const float* __restrict__ w, int H, int E, long stride, float eps) {
  __shared__ float scratch[4];
  const long t = blockIdx.x;
  const int h = blockIdx.y;
  const float* op = o + (t * H + h) * E;
  float ss = 0.f;
  for (int e = threadIdx.x; e < E; e += 256) ss += op[e] * op[e];
  ss = block_reduce_sum_256(ss, scratch);
  const float rs = 1.f / sqrtf(ss / E + eps);
  for (int e = threadIdx.x; e < E; e += 256)
    Elem<T>::st(y + (t * H + h) * E + e,
                op[e] * rs * w[K == MLSTM ? h * E + e : e] *
                    out_gate<T, K>(
                        Elem<T>::ld(g + t * stride + (long)h * E + e)));
}

// ---- decode step ----------------------------------------------------------
// One workgroup per (sequence, head, `cols` columns): reads and writes its
// part of the head's state once.  A kind with a norm per head needs all E
// columns; lightning attention writes o itself, float, and may divide them.
// Thread t covers V columns starting at (t % LPR) * V (and every LPR * V on)
// in rows t / LPR + i * R; partial sums over rows meet in LDS.
template <typename T, int V, Kind K>
__global__ __launch_bounds__(256) void recurrent_step_kernel(
    T* __restrict__ y, float* __restrict__ o_raw, float* __restrict__ S,
    float* __restrict__ n_pool, float* __restrict__ m_pool,
    const T* __restrict__ q, const T* __restrict__ k,
    const T* __restrict__ v, const T* __restrict__ g,
    const T* __restrict__ a1h,
    const T* __restrict__ a2, const float* __restrict__ b0,
    const float* __restrict__ b1, const float* __restrict__ raw,
    const float* __restrict__ w, const long* __restrict__ positions,
    const int* __restrict__ slots, int H, int D, int E, int cols, int rank,
    long stride, float qscale, float tau_or_cap, float eps) {
  extern __shared__ float sm[];
  float* qd = sm;                    // [D]
  float* kd = sm + D;                // [D]
  float* ad = sm + 2 * D;            // [D] decay (GLA)
  float* part = sm + 3 * D;          // [R][cols] partial o
  __shared__ float scratch[4];
  const long row = blockIdx.x;
  const int h = blockIdx.y;
  const int tid = threadIdx.x;
  const int slot = slots[row];
  const bool fresh = slot < 0 || positions[row] == 0;
  const int c0 = blockIdx.z * cols, cn = min(cols, E - c0);
  const int LPR = min(cols / V, 256);
  const int R = 256 / LPR;
  const int r0 = tid / LPR;

  float fs = K == LIGHTNING ? b0[h] : 1.f, is = 1.f, m = 0.f;
  if constexpr (K == MLSTM) {
    float li, lf;
    mlstm_gates(raw[row * 2 * H + h] + b0[h], raw[row * 2 * H + H + h] + b1[h],
                tau_or_cap, &li, &lf);
    const float mo = fresh ? 0.f : m_pool[(long)slot * H + h];
    m = fmaxf(lf + mo, li);
    fs = expf(lf + mo - m);
    is = expf(li - m);
  }
  float den = 0.f;
  for (int d = tid; d < D; d += 256) {
    const long at = row * stride + (long)h * D + d;
    const float qv = entry<T, K>(q + at) * qscale;
    const float kv = entry<T, K>(k + at) * is;
    qd[d] = qv;
    kd[d] = kv;
    if constexpr (K == MLSTM) {
      float* np = n_pool + ((long)max(slot, 0) * H + h) * D + d;
      const float n = (fresh ? 0.f : *np * fs) + kv;
      if (slot >= 0) *np = n;
      den += n * qv;
    }
  }
  if constexpr (K == GLA) {
    // four lanes a channel share the inner product of its decay
    for (int u = tid; u < 4 * D; u += 256) {
      const int c = h * D + (u >> 2);
      float z = (u & 3) == 0 ? b0[c] : 0.f;
      #pragma unroll 4
      for (int r = u & 3; r < rank; r += 4)
        z += Elem<T>::ld(a1h + row * stride + r) *
             Elem<T>::ld(a2 + (long)c * rank + r);
      z += __shfl_xor(z, 1);
      z += __shfl_xor(z, 2);
      if ((u & 3) == 0) ad[u >> 2] = expf(log_sigmoid(z) / tau_or_cap);
    }
  }
  float inv = 1.f;
  if constexpr (K == MLSTM) {
    den = block_reduce_sum_256(den, scratch);
    inv = 1.f / (fmaxf(fabsf(den), expf(-m)) + DEN_EPS);
    if (slot >= 0 && tid == 0) m_pool[(long)slot * H + h] = m;
  }
  __syncthreads();

  for (int e = (tid % LPR) * V; r0 < R && e < cn; e += LPR * V) {
    float acc[V] = {};
    float vv[V];
    load_vec<T, V>(v + row * stride + (long)h * E + c0 + e, vv);
    if constexpr (K == LIGHTNING) {
      #pragma unroll
      for (int i = 0; i < V; ++i) vv[i] /= 1.f + Fn<T>::exp(-vv[i]);
    }
    float* Sp = S + ((long)max(slot, 0) * H + h) * D * E + c0 + e;
    #pragma unroll 8
    for (int d = r0; d < D; d += R) {
      float s[V] = {};
      if (!fresh) load_vec<float, V>(Sp + (long)d * E, s);
      const float a = K == GLA ? ad[d] : fs;
      const float kv = kd[d], qv = qd[d];
      #pragma unroll
      for (int i = 0; i < V; ++i) {
        s[i] = s[i] * a + kv * vv[i];
        acc[i] += s[i] * qv;
      }
      if (slot >= 0) store_vec<float, V>(Sp + (long)d * E, s);
    }
    #pragma unroll
    for (int i = 0; i < V; ++i) part[r0 * cols + e + i] = acc[i];
  }
  __syncthreads();
  float ss = 0.f;
  for (int c = tid; c < cn; c += 256) {
    float o = 0.f;
    for (int r = 0; r < R; ++r) o += part[r * cols + c];
    if constexpr (K == LIGHTNING) {
      o_raw[(row * H + h) * E + c0 + c] = o;
    } else {
      o *= inv;
      part[c] = o;                    // row 0 is read by this thread only
      ss += o * o;
    }
  }
  if constexpr (K == LIGHTNING) return;
  ss = block_reduce_sum_256(ss, scratch);
  const float rs = 1.f / sqrtf(ss / E + eps);
  for (int c = tid; c < E; c += 256)
    Elem<T>::st(y + (row * H + h) * E + c,
                part[c] * rs * w[K == MLSTM ? h * E + c : c] *
                    out_gate<T, K>(
                        Elem<T>::ld(g + row * stride + (long)h * E + c)));
}

}  // namespace

template <typename T>
void launch_gla_decay(float* log_decay, const T* a1h, const T* a2,
                      const float* a2b, long rows, int channels, int rank,
                      float tau, long stride, hipStream_t stream) {
  if (rows == 0) return;
  gla_decay_kernel<T><<<dim3((unsigned)rows,
                             (unsigned)((channels + 255) / 256)),
                        256, 0, stream>>>(log_decay, a1h, a2, a2b, channels,
                                          rank, 1.f / tau, stride);
}

void launch_mlstm_gates(float* out, const float* raw, const float* ib,
                        const float* fb, long rows, int H, float cap,
                        hipStream_t stream) {
  if (rows == 0) return;
  mlstm_gates_kernel<<<dim3((unsigned)((rows * H + 255) / 256)), 256, 0,
                       stream>>>(out, raw, ib, fb, rows, H, cap);
}

// gates: log decays [T, H, D], log gates [T, 2H] or decays [H], by kind
template <typename T>
void launch_recurrent_scan(Kind kind, float* o, float* S, float* n_pool, float* m_pool,
                           float* nm_new, const T* q, const T* k, const T* v,
                           const float* gates, const int* seq_start,
                           const long* positions, const int* slots,
                           int num_seqs, int H, int D, int E, long stride,
                           float qscale, hipStream_t stream) {
  if (num_seqs == 0) return;
  const dim3 grid((unsigned)((E + COLS - 1) / COLS), (unsigned)H,
                  (unsigned)num_seqs);
  #define SCAN(RPL)                                                         \
    if (D <= 64 * RPL) {                                                    \
      if (kind == MLSTM) RUN(RPL, MLSTM);                                   \
      else if (kind == GLA) RUN(RPL, GLA);                                  \
      else RUN(RPL, LIGHTNING);                                             \
    }
  #define RUN(RPL, K)                                                       \
    recurrent_scan_kernel<T, RPL, K><<<grid, 64, 0, stream>>>(              \
        o, S, n_pool, m_pool, nm_new, q, k, v, gates, seq_start, positions, \
        slots, H, D, E, stride, qscale)
  if (D > 1024)
    throw std::runtime_error("recurrent_scan: key size above 1024");
  SCAN(1) else SCAN(2) else SCAN(4) else SCAN(8) else SCAN(16)
  #undef RUN
  #undef SCAN
  if (kind == MLSTM)
    mlstm_commit_kernel<<<dim3((unsigned)H, (unsigned)num_seqs), 256, 0,
                          stream>>>(n_pool, m_pool, nm_new, seq_start, slots,
                                    H, D);
}

template <typename T>
void launch_recurrent_out(T* y, const float* o, const T* g, const float* w,
                          bool mlstm, long rows, int H, int E, long stride,
                          float eps, hipStream_t stream) {
  if (rows == 0) return;
  const dim3 grid((unsigned)rows, (unsigned)H);
  if (mlstm)
    recurrent_out_kernel<T, MLSTM><<<grid, 256, 0, stream>>>(y, o, g, w, H, E,
                                                            stride, eps);
  else
    recurrent_out_kernel<T, GLA><<<grid, 256, 0, stream>>>(y, o, g, w, H, E,
                                                             stride, eps);
}

template <typename T>
void launch_recurrent_step(Kind kind, T* y, float* o_raw, float* S,
                           float* n_pool, float* m_pool, const T* q,
                           const T* k, const T* v, const T* g, const T* a1h,
                           const T* a2, const float* b0, const float* b1,
                           const float* raw, const float* w,
                           const long* positions, const int* slots,
                           long rows, int H, int D, int E, int rank,
                           long stride, float qscale, float tau_or_cap,
                           float eps, hipStream_t stream) {
  if (rows == 0) return;
  // four columns a thread needs 16-byte aligned rows of every operand
  const bool vec = E % 4 == 0 && stride % 4 == 0 &&
                   (reinterpret_cast<uintptr_t>(v) % (4 * sizeof(T))) == 0;
  int cols = E;
  if (kind == LIGHTNING)              // small batches: fill the chip
    while (rows * H * (E / cols) < 512 && cols % 8 == 0 && cols >= 64)
      cols /= 2;
  const dim3 grid((unsigned)rows, (unsigned)H,
                  (unsigned)((E + cols - 1) / cols));
  #define STEP(V, K)                                                        \
    recurrent_step_kernel<T, V, K>                                          \
        <<<grid, 256, (3 * D + max(256 * V, cols)) * sizeof(float),         \
           stream>>>(y, o_raw, S, n_pool, m_pool, q, k, v, g, a1h, a2, b0,  \
                     b1, raw, w, positions, slots, H, D, E, cols, rank,     \
                     stride, qscale, tau_or_cap, eps)
  #define STEP_KIND(K)                                                      \
    if (kind == K) {                                                        \
      if (vec) STEP(4, K); else STEP(1, K);                                 \
    }
  STEP_KIND(GLA) STEP_KIND(MLSTM) STEP_KIND(LIGHTNING)
  #undef STEP_KIND
  #undef STEP
}

#define INSTANTIATE(T)                                                      \
  template void launch_gla_decay<T>(float*, const T*, const T*,             \
                                    const float*, long, int, int, float,    \
                                    long, hipStream_t);                     \
  template void launch_recurrent_scan<T>(                                   \
      Kind, float*, float*, float*, float*, float*, const T*, const T*, const T*, \
      const float*, const int*, const long*, const int*, int, int, int,     \
      int, long, float, hipStream_t);                                       \
  template void launch_recurrent_out<T>(T*, const float*, const T*,         \
                                        const float*, bool, long, int, int, \
                                        long, float, hipStream_t);          \
  template void launch_recurrent_step<T>(                                   \
      Kind, T*, float*, float*, float*, float*, const T*, const T*,         \
      const T*, const T*, const T*, const T*, const float*, const float*,   \
      const float*, const float*, const long*, const int*, long, int, int,  \
      int, int, long, float, float, float, hipStream_t);
INSTANTIATE(bf16)
INSTANTIATE(float)
#undef INSTANTIATE
