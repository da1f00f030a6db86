// Windowed latent attention over the paged cache (gfx950).
//
// A token keeps one row [c (rank) | k_r (rot)] for all heads, c normed and
// k_r rotated:                      cache [NB, 16, rank + rot]
// Head h has k = [W_uk[h] c | k_r], v = W_uv[h] c and
//   score(i, j) = (q_i . k_j) * scale,  i - window < j <= i.
// The softmax denominator of head h also has exp(sink[h]), once, without a
// value, and the head's output is multiplied by sigmoid(gate[i, h]) (null:
// nothing).
//
//   q   [T, H, D + rot]  (token stride qs), the last rot of a head rotated
//   uk  [rank, H * D]    (W_uk transposed)    uv [H * E, rank]
//
// Absorbed: qa = W_uk^T q_unrotated per head (head_gemm), attention of
// [qa | q_r] over the rows themselves giving sum_j p_j c_j, then W_uv
// (head_gemm).  Expanded: k and v of the visible rows are formed per head
// with plain products, v transposed, and attended like ordinary ones.
//
// Matrix-core kernels (bf16): sizes are multiples of 8, padded with zeros in
// registers and LDS.  The attention weights enter as a bf16 high and low
// part.  Scores are formed transposed, S^T = K Q^T, so that a lane holds one
// query column.  The general kernels take any sizes, bf16 or float.
#include <float.h>

#include <algorithm>

#include "rotary.h"
#include "side.h"

#define PAGE 16

typedef __attribute__((ext_vector_type(4))) short short4_t;

namespace {

constexpr float LOG2E = 1.4426950408889634f;

DEV float exp2_fast(float x) { return __builtin_amdgcn_exp2f(x); }

// ---- rotation of q, norm and rotation of a token's row, append -----------
// One workgroup a token, blockIdx.y 0; the others have an activation of the
// same rows.  freqs holds the angle per position of every pair; cosine and
// sine are multiplied by `gain`.
template <typename T, int V>
__global__ __launch_bounds__(256) void latent_rope_append_kernel(
    T* __restrict__ q, const T* __restrict__ kv, const float* __restrict__ w,
    const long* __restrict__ positions, const double* __restrict__ freqs,
    const long* __restrict__ slot_mapping, T* __restrict__ cache, int H,
    int D, int rank, int rot, long qs, long ks, float eps, float gain,
    SideRelu<T> side) {
  extern __shared__ float cs[];        // (cos, sin) of each pair
  __shared__ float scratch[4];
  const long row = blockIdx.x;
  if (blockIdx.y > 0) {
    side_relu(side, row, 1, blockIdx.y - 1);
    return;
  }
  const int half = rot / 2;
  for (int i = threadIdx.x; i < half; i += 256) {
    float c, s;
    angle<T>(positions[row], freqs[i], &c, &s);
    cs[2 * i] = c * gain;
    cs[2 * i + 1] = s * gain;
  }
  __syncthreads();
  // W elements of a head at a time
  constexpr int W = V == 1 ? 2 : V;
  const int units = rot / W;
  for (int u = threadIdx.x; u < H * units; u += 256) {
    const int h = u / units, d = u % units * W;
    T* p = q + row * qs + (long)h * (D + rot) + D + d;
    float x[W];
    if constexpr (V == 1) {
      x[0] = Elem<T>::ld(p);
      x[1] = Elem<T>::ld(p + 1);
    } else {
      load_vec<T, V>(p, x);
    }
    turn_pairs<W>(x, cs + d);
    if constexpr (V == 1) {
      Elem<T>::st(p, x[0]);
      Elem<T>::st(p + 1, x[1]);
    } else {
      store_vec<T, V>(p, x);
    }
  }
  if (!kv) return;
  const long slot = slot_mapping[row];
  if (slot < 0) return;                // the whole workgroup
  const T* src = kv + row * ks;
  T* dst = cache + slot * (rank + rot);
  float ss = 0.f;
  for (int c = threadIdx.x * V; c < rank; c += 256 * V) {
    float f[V];
    load_vec<T, V>(src + c, f);
    #pragma unroll
    for (int i = 0; i < V; ++i) ss += f[i] * f[i];
  }
  ss = block_reduce_sum_256(ss, scratch);
  const float rs = 1.f / sqrtf(ss / rank + eps);
  for (int c = threadIdx.x * V; c < rank; c += 256 * V) {
    float f[V], wv[V];
    load_vec<T, V>(src + c, f);
    load_vec<float, V>(w + c, wv);
    #pragma unroll
    for (int i = 0; i < V; ++i) f[i] *= rs * wv[i];
    store_vec<T, V>(dst + c, f);
  }
  for (int i = threadIdx.x; i < half; i += 256) {
    float x[2] = {Elem<T>::ld(src + rank + 2 * i),
                  Elem<T>::ld(src + rank + 2 * i + 1)};
    turn_pairs<2>(x, cs + 2 * i);
    Elem<T>::st(dst + rank + 2 * i, x[0]);
    Elem<T>::st(dst + rank + 2 * i + 1, x[1]);
  }
}

// rows of the cache by slot, in units of 8 elements; slot -1 gives zeros
__global__ __launch_bounds__(256) void latent_gather_kernel(
    uint4* __restrict__ out, const uint4* __restrict__ cache,
    const long* __restrict__ slots, long total, int units) {
  const long u = (long)blockIdx.x * 256 + threadIdx.x;
  if (u >= total) return;
  const long row = u / units;
  const long slot = slots[row];
  out[u] = slot < 0 ? uint4{0, 0, 0, 0} : cache[slot * units + u % units];
}

// ---- a small product per head ---------------------------------------------
// sigmoid(g[row, h]), null: 1
template <typename T> struct Gate {
  const T* g;
  long stride;

  DEV float operator()(long row, int h) const {
    return g ? 1.f / (1.f + Fn<T>::exp(-Elem<T>::ld(g + row * stride + h)))
             : 1.f;
  }
};

// out[r, h, n] = sum_k x[r, h, k] w[h, n, k] with strides, times the gate of
// out's row; `rows_in` and `rows_out` map r to rows of x and out (null: r
// itself)
struct HeadGemm {
  const int* rows_in;
  const int* rows_out;
  long R;
  int N, K;
  long xr, xh, wn, wh, outr, outh;
};

template <typename T>
__global__ __launch_bounds__(256) void head_gemm_general_kernel(
    T* __restrict__ out, const T* __restrict__ x, const T* __restrict__ w,
    HeadGemm a, Gate<T> gate) {
  const long r = blockIdx.x;
  const int h = blockIdx.y, lane = threadIdx.x & 63;
  const T* xp = x + (a.rows_in ? a.rows_in[r] : r) * a.xr + h * a.xh;
  const long row = a.rows_out ? a.rows_out[r] : r;
  T* op = out + row * a.outr + h * a.outh;
  const float f = gate(row, h);
  for (int n = threadIdx.x >> 6; n < a.N; n += 4) {
    const T* wp = w + h * a.wh + n * a.wn;
    float s = 0.f;
    for (int k = lane; k < a.K; k += 64)
      s += Elem<T>::ld(xp + k) * Elem<T>::ld(wp + k);
    s = wave_reduce_sum(s);
    if (lane == 0) Elem<T>::st(op + n, s * f);
  }
}

// a wave has 16 n and CT tiles of 16 rows
template <int CT>
__global__ __launch_bounds__(256) void head_gemm_kernel(
    bf16* __restrict__ out, const bf16* __restrict__ x,
    const bf16* __restrict__ w, HeadGemm a, Gate<bf16> gate) {
  const int lane = threadIdx.x & 63, col = lane & 15, gr = lane >> 4;
  const int n0 = (blockIdx.x * 4 + (threadIdx.x >> 6)) * 16;
  const int h = blockIdx.z;
  if (n0 >= a.N) return;
  const bool wn = n0 + col < a.N;
  const bf16* wp = w + h * a.wh + (long)(n0 + col) * a.wn + gr * 8;
  const bf16* xp[CT];
  bool live[CT];
  #pragma unroll
  for (int t = 0; t < CT; ++t) {
    const long r = ((long)blockIdx.y * CT + t) * 16 + col;
    live[t] = r < a.R;
    xp[t] = x + (live[t] && a.rows_in ? a.rows_in[r] : r) * a.xr + h * a.xh +
            gr * 8;
  }
  f32x4_t acc[CT];
  #pragma unroll
  for (int t = 0; t < CT; ++t) acc[t] = f32x4_t(0.f);
  #pragma unroll 8
  for (int k = 0; k < a.K; k += 32) {
    const bool in = k + gr * 8 < a.K;
    const short8_t wf = in && wn
        ? *reinterpret_cast<const short8_t*>(wp + k) : short8_t{};
    #pragma unroll
    for (int t = 0; t < CT; ++t) {
      const short8_t xf = in && live[t]
          ? *reinterpret_cast<const short8_t*>(xp[t] + k) : short8_t{};
      acc[t] = mfma16(wf, xf, acc[t]);
    }
  }
  const int n = n0 + gr * 4;
  if (n >= a.N) return;                 // N is a multiple of 8
  #pragma unroll
  for (int t = 0; t < CT; ++t) {
    if (!live[t]) continue;
    const long r = ((long)blockIdx.y * CT + t) * 16 + col;
    const long row = a.rows_out ? a.rows_out[r] : r;
    const float f = gate(row, h);
    *reinterpret_cast<uint2*>(out + row * a.outr + h * a.outh + n) =
        uint2{cvt_pk_bf16(acc[t][0] * f, acc[t][1] * f),
              cvt_pk_bf16(acc[t][2] * f, acc[t][3] * f)};
  }
}

// ---- absorbed attention, any sizes ----------------------------------------
constexpr int TILE = 256;      // tokens per softmax step
constexpr int MAX_RPT = 8;     // latent columns a thread: rank <= 2048

template <typename T>
__global__ __launch_bounds__(256) void latent_attn_general_kernel(
    T* __restrict__ out, const T* __restrict__ qa, const T* __restrict__ q,
    const T* __restrict__ cache, const int* __restrict__ block_tables,
    const long* __restrict__ positions, const int* __restrict__ rows,
    const int* __restrict__ row_seq, const float* __restrict__ sink,
    int max_blocks, int H, int D, int rank, int rot, int window, float scale,
    long qs) {
  extern __shared__ float general_lds[];
  const int width = rank + rot;
  float* q_lds = general_lds;          // [width]
  float* p_lds = q_lds + width;        // [TILE]
  __shared__ float scratch[4];
  const long r = blockIdx.x;
  const int h = blockIdx.y, tid = threadIdx.x;
  const long row = rows ? rows[r] : r;
  const int* bt = block_tables +
                  (long)(row_seq ? row_seq[row] : (int)row) * max_blocks;
  const long pos = positions[row];
  const long lo = pos - window + 1 > 0 ? pos - window + 1 : 0;
  for (int i = tid; i < width; i += 256)
    q_lds[i] = i < rank
        ? Elem<T>::ld(qa + (r * H + h) * rank + i)
        : Elem<T>::ld(q + row * qs + (long)h * (D + rot) + D + i - rank);
  __syncthreads();
  float acc[MAX_RPT] = {};
  float m = sink ? sink[h] : -FLT_MAX, l = sink ? 1.f : 0.f;
  for (long base = lo; base <= pos; base += TILE) {
    const int n = (int)min((long)TILE, pos - base + 1);
    float s = -FLT_MAX;
    if (tid < n) {
      const long p = base + tid;
      const T* kp = cache + ((long)bt[p / PAGE] * PAGE + p % PAGE) * width;
      float d = 0.f;
      for (int i = 0; i < width; ++i) d += q_lds[i] * Elem<T>::ld(kp + i);
      s = d * scale;
    }
    const float mn = fmaxf(m, block_reduce_max_256(s, scratch));
    const float p = tid < n ? Fn<T>::exp(s - mn) : 0.f;
    const float alpha = m == -FLT_MAX ? 0.f : Fn<T>::exp(m - mn);
    l = l * alpha + block_reduce_sum_256(p, scratch);
    m = mn;
    p_lds[tid] = p;
    __syncthreads();
    #pragma unroll
    for (int i = 0; i < MAX_RPT; ++i) {
      const int e = tid + 256 * i;
      if (e < rank) {
        float a = acc[i] * alpha;
        for (int t = 0; t < n; ++t) {
          const long pt = base + t;
          a += p_lds[t] * Elem<T>::ld(
              cache + ((long)bt[pt / PAGE] * PAGE + pt % PAGE) * width + e);
        }
        acc[i] = a;
      }
    }
    __syncthreads();
  }
  #pragma unroll
  for (int i = 0; i < MAX_RPT; ++i)
    if (tid + 256 * i < rank)
      Elem<T>::st(out + (r * H + h) * rank + tid + 256 * i, acc[i] / l);
}

// ---- absorbed attention, matrix cores -------------------------------------
// A workgroup has one row, HT tiles of 16 heads and every split-th tile of
// KT tokens.  A tile is staged once in LDS (two buffers): the score product
// reads it row by row, the value product reads its transpose with the
// transposing LDS load.  In the score product wave w has tokens
// (w & 1) * 16 and head tile w >> 1 (one head tile: half of the columns); in
// the value product every wave has all heads and a quarter of the latent.
constexpr int KT = 32;
constexpr int SS = KT + 4;         // row of the score tile

// four rows of one column: in every 16 lanes, lane i passes the address of
// row i / 4, columns 4 (i % 4), and receives column i
DEV short4_t lds_read_tr(const short* p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16(
      (__attribute__((address_space(3))) short4_t*)p);
}

constexpr int decode_lds(int RP, int XP) {
  return 2 * KT * (RP + XP + 8) * 2 + 2 * 16 * SS * 4;
}

// EXACT: rank == RP and rot == XP, a row is staged as it is
template <int RP, int XP, int HT, bool EXACT>
__global__ __launch_bounds__(256, 2) void latent_attn_decode_kernel(
    bf16* __restrict__ out, float* __restrict__ partial,
    const bf16* __restrict__ qa, const bf16* __restrict__ q,
    const bf16* __restrict__ cache, const int* __restrict__ block_tables,
    const long* __restrict__ positions, const int* __restrict__ rows,
    const int* __restrict__ row_seq, const float* __restrict__ sink,
    int max_blocks, int H, int D, int rank, int rot, int window, float scale2,
    long qs) {
  constexpr int LS = RP + XP + 8;            // row of a staged tile
  constexpr int KC = (RP + XP) / 32;         // steps of the score product
  constexpr int QC = HT == 2 ? KC : (KC + 1) / 2;
  constexpr int ET = RP / 64;                // 16-column tiles of a wave
  constexpr int UPR = (RP + XP) / 8;         // 16-byte units of a row
  constexpr int LOADS = (UPR + 7) / 8;       // units a thread: 8 share a row
  extern __shared__ __attribute__((aligned(16))) char smem[];
  short* kv_lds = reinterpret_cast<short*>(smem);            // [2][KT][LS]
  float* s_lds = reinterpret_cast<float*>(kv_lds + 2 * KT * LS);

  const long r = blockIdx.x;
  const int h0 = blockIdx.y * HT * 16;
  const int split = gridDim.z, z = blockIdx.z;
  const long row = rows ? rows[r] : r;
  const int* bt = block_tables +
                  (long)(row_seq ? row_seq[row] : (int)row) * max_blocks;
  const int pos = (int)positions[row];
  const int lo = max(0, pos - window + 1);
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int col = lane & 15, gr = lane >> 4;
  const int tg = wid & 1, part = wid >> 1;

  // this wave's query columns: steps [c0, c0 + QC) of head tile `part`
  const int c0 = HT == 2 ? 0 : part * QC;
  short8_t qf[QC];
  {
    const int h = h0 + (HT == 2 ? part * 16 : 0) + col;
    #pragma unroll
    for (int c = 0; c < QC; ++c) {
      const int d = (c0 + c) * 32 + gr * 8;
      qf[c] = short8_t{};
      if (h < H) {
        if (d < RP) {
          if (d < rank)
            qf[c] = *reinterpret_cast<const short8_t*>(
                qa + (r * H + h) * rank + d);
        } else if (d - RP < rot) {
          qf[c] = *reinterpret_cast<const short8_t*>(
              q + row * qs + (long)h * (D + rot) + D + d - RP);
        }
      }
    }
  }
  f32x4_t acc[HT][ET];
  #pragma unroll
  for (int t = 0; t < HT; ++t)
    #pragma unroll
    for (int e = 0; e < ET; ++e) acc[t][e] = f32x4_t(0.f);
  float m[HT], l[HT];
  #pragma unroll
  for (int t = 0; t < HT; ++t) {
    m[t] = -FLT_MAX;
    l[t] = 0.f;
    if (sink && z == 0) {            // counted once: by a quarter of the lanes
      m[t] = sink[min(h0 + t * 16 + col, H - 1)] * LOG2E;
      l[t] = gr == 0 ? 1.f : 0.f;
    }
  }

  // This thread stages units tid % 8 + 8 i of token tid / 8.  Tokens past the
  // row's own read its own again (their weight is zero); padding columns are
  // zeros.  A page id is read one tile ahead of its rows.
  const int tok = tid >> 3;
  int off[LOADS];                    // column in the cache row, -1: zeros
  #pragma unroll
  for (int i = 0; i < LOADS; ++i) {
    const int d = ((tid & 7) + 8 * i) * 8;
    off[i] = d < RP ? (d < rank ? d : -1)
                    : d - RP < rot ? d - RP + rank : -1;
  }
  short8_t kr[LOADS];
  long page = 0;
  auto fetch = [&](int p0) {
    const int p = min(p0 + tok, pos);
    const bf16* src = cache + (page * PAGE + p % PAGE) * (rank + rot);
    page = bt[min(p0 + split * KT + tok, pos) / PAGE];
    #pragma unroll
    for (int i = 0; i < LOADS; ++i) {
      if constexpr (EXACT)
        kr[i] = *reinterpret_cast<const short8_t*>(src + (tid & 7) * 8 +
                                                   64 * i);
      else
        kr[i] = off[i] >= 0 ? *reinterpret_cast<const short8_t*>(src + off[i])
                            : short8_t{};
    }
  };

  int p0 = (lo / KT + z) * KT, buf = 0;
  if (p0 <= pos) {
    page = bt[min(p0 + tok, pos) / PAGE];
    fetch(p0);
  }
  for (; p0 <= pos; p0 += split * KT, buf ^= 1) {
    short* tile = kv_lds + buf * KT * LS;
    #pragma unroll
    for (int i = 0; i < LOADS; ++i)
      if ((tid & 7) + 8 * i < UPR)
        *reinterpret_cast<short8_t*>(tile + tok * LS + (tid & 7) * 8 +
                                     64 * i) = kr[i];
    __syncthreads();
    if (p0 + split * KT <= pos) fetch(p0 + split * KT);
    {
      f32x4_t sc = f32x4_t(0.f);
      #pragma unroll
      for (int c = 0; c < QC; ++c)
        if (c0 + c < KC)
          sc = mfma16(*reinterpret_cast<const short8_t*>(
                          tile + (tg * 16 + col) * LS + (c0 + c) * 32 +
                          gr * 8),
                      qf[c], sc);
      *reinterpret_cast<f32x4_t*>(
          s_lds + (part * 16 + col) * SS + tg * 16 + gr * 4) = sc;
    }
    __syncthreads();
    short8_t ph[HT], pl[HT];
    const bool full = p0 >= lo && p0 + KT - 1 <= pos;
    #pragma unroll
    for (int t = 0; t < HT; ++t) {
      float p[8], mx = m[t];
      const float* sp = s_lds + (t * 16 + col) * SS + gr * 8;
      *reinterpret_cast<float4*>(p) = *reinterpret_cast<const float4*>(sp);
      *reinterpret_cast<float4*>(p + 4) =
          *reinterpret_cast<const float4*>(sp + 4);
      if constexpr (HT == 1) {
        #pragma unroll
        for (int i = 0; i < 8; ++i) p[i] += sp[16 * SS + i];
      }
      #pragma unroll
      for (int i = 0; i < 8; ++i) p[i] *= scale2;
      if (!full) {
        #pragma unroll
        for (int i = 0; i < 8; ++i) {
          const int at = p0 + gr * 8 + i;
          if (at < lo || at > pos) p[i] = -FLT_MAX;
        }
      }
      #pragma unroll
      for (int i = 0; i < 8; ++i) mx = fmaxf(mx, p[i]);
      mx = fmaxf(mx, __shfl_xor(mx, 16));
      mx = fmaxf(mx, __shfl_xor(mx, 32));
      if (!__all(mx == m[t])) {
        const float alpha = m[t] == -FLT_MAX ? 0.f : exp2_fast(m[t] - mx);
        #pragma unroll
        for (int e = 0; e < ET; ++e)
          #pragma unroll
          for (int i = 0; i < 4; ++i) acc[t][e][i] *= alpha;
        l[t] *= alpha;
        m[t] = mx;
      }
      const float base = m[t] == -FLT_MAX ? 0.f : m[t];
      #pragma unroll
      for (int i = 0; i < 8; ++i) {
        p[i] = exp2_fast(p[i] - base);
        l[t] += p[i];
      }
      split_bf16x8(p, &ph[t], &pl[t]);
    }
    const short* vp = tile + (gr * 8 + (col >> 2)) * LS + wid * (RP / 4) +
                      (col & 3) * 4;
    #pragma unroll
    for (int e = 0; e < ET; ++e) {
      const short4_t a = lds_read_tr(vp + e * 16);
      const short4_t b = lds_read_tr(vp + 4 * LS + e * 16);
      const short8_t vf{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
      #pragma unroll
      for (int t = 0; t < HT; ++t) {
        acc[t][e] = mfma16(vf, ph[t], acc[t][e]);
        acc[t][e] = mfma16(vf, pl[t], acc[t][e]);
      }
    }
  }
  #pragma unroll
  for (int t = 0; t < HT; ++t) {
    l[t] += __shfl_xor(l[t], 16);
    l[t] += __shfl_xor(l[t], 32);
    const int h = h0 + t * 16 + col;
    if (h >= H) continue;
    const float f = split > 1 ? 1.f : 1.f / l[t];
    const long at = split > 1
        ? ((r * H + h) * split + z) * (rank + 4) : (r * H + h) * rank;
    #pragma unroll
    for (int e = 0; e < ET; ++e) {
      const int d = wid * (RP / 4) + e * 16 + gr * 4;
      if (d >= rank) continue;
      if (split > 1)
        *reinterpret_cast<f32x4_t*>(partial + at + d) = acc[t][e];
      else
        *reinterpret_cast<uint2*>(out + at + d) =
            uint2{cvt_pk_bf16(acc[t][e][0] * f, acc[t][e][1] * f),
                  cvt_pk_bf16(acc[t][e][2] * f, acc[t][e][3] * f)};
    }
    if (split > 1 && wid == 0 && gr == 0) {
      partial[at + rank] = m[t];
      partial[at + rank + 1] = l[t];
    }
  }
}

// Partial results of RB <= 16 rows and one head combined, then W_uv of that
// head: out[row, h] = W_uv[h] sum_p weight_p o_p.  split <= 16, rank <= 512.
// NW waves, 4 or 8; a wave has 16 of every gridDim.z * NW * 16 values, its
// first weights are on their way while the results are combined.
template <int RB, int NW>
__global__ __launch_bounds__(64 * NW) void latent_merge_values_kernel(
    bf16* __restrict__ out, const float* __restrict__ partial,
    const bf16* __restrict__ uv, const int* __restrict__ rows, long R,
    int split, int H, int E, int rank, long os, Gate<bf16> gate) {
  extern __shared__ __attribute__((aligned(16))) short merged[];
  __shared__ float weight[16][17];
  constexpr int GROUPS = NW / 4;             // of waves, each has other rows
  constexpr int RG = RB < GROUPS ? 1 : RB / GROUPS;
  constexpr int RK = RG < 4 ? RG : 4;        // rows combined together
  const int h = blockIdx.y, tid = threadIdx.x;
  const long r0 = (long)blockIdx.x * RB;
  const int live = (int)min((long)RB, R - r0);
  const int XS = rank + 8;
  const int lane = tid & 63, wid = tid >> 6, col = lane & 15, gr = lane >> 4;
  int n0 = (blockIdx.z * NW + wid) * 16;
  short8_t wf[16];
  auto weights = [&]() {
    const bool wn = n0 + col < E;
    const bf16* wp = uv + ((long)h * E + n0 + col) * rank + gr * 8;
    #pragma unroll
    for (int k = 0; k < 16; ++k)
      wf[k] = wn && k * 32 + gr * 8 < rank
          ? *reinterpret_cast<const short8_t*>(wp + k * 32) : short8_t{};
  };
  weights();
  const long r = rows && col < live ? rows[r0 + col] : r0 + col;
  const float f = col < live ? gate(r, h) : 0.f;
  if (tid < 256) {
    const int i = tid >> 4, p = tid & 15;
    const bool in = i < live && p < split;
    const float* src = partial +
        (((r0 + i) * H + h) * split + p) * (rank + 4) + rank;
    const float m = in ? src[0] : -FLT_MAX, l = in ? src[1] : 0.f;
    float mx = m;
    #pragma unroll
    for (int o = 1; o < 16; o <<= 1) mx = fmaxf(mx, __shfl_xor(mx, o));
    const float w = m == -FLT_MAX ? 0.f : exp2_fast(m - mx);
    float sum = w * l;
    #pragma unroll
    for (int o = 1; o < 16; o <<= 1) sum += __shfl_xor(sum, o);
    weight[i][p] = sum > 0.f ? w / sum : 0.f;
  }
  __syncthreads();
  // a wave has a quarter of the columns
  const int quarter = rank / 4, part = wid & 3;
  for (int c = part * quarter + lane * 2; c < (part + 1) * quarter; c += 128)
    for (int i0 = (wid >> 2) * RK; i0 < live; i0 += GROUPS * RK) {
      float2 o[RK] = {};
      const float* src[RK];
      #pragma unroll
      for (int k = 0; k < RK; ++k)
        src[k] = partial + ((r0 + min(i0 + k, live - 1)) * H + h) * split *
                               (rank + 4) + c;
      #pragma unroll 8
      for (int p = 0; p < split; ++p)
        #pragma unroll
        for (int k = 0; k < RK; ++k) {
          const float w = weight[i0 + k][p];
          const float2 x = *reinterpret_cast<const float2*>(
              src[k] + (long)p * (rank + 4));
          o[k].x += w * x.x;
          o[k].y += w * x.y;
        }
      #pragma unroll
      for (int k = 0; k < RK; ++k)
        *reinterpret_cast<unsigned*>(merged + (i0 + k) * XS + c) =
            cvt_pk_bf16(o[k].x, o[k].y);
    }
  __syncthreads();
  while (n0 < E) {
    f32x4_t acc = f32x4_t(0.f);
    #pragma unroll
    for (int k = 0; k < 16; ++k) {
      if (k * 32 >= rank) break;
      // columns past the last row are left out below
      const short8_t xf = k * 32 + gr * 8 < rank && col < live
          ? *reinterpret_cast<const short8_t*>(merged + col * XS + k * 32 +
                                               gr * 8)
          : short8_t{};
      acc = mfma16(wf[k], xf, acc);
    }
    const int n = n0 + gr * 4;
    if (n < E && col < live)
      *reinterpret_cast<uint2*>(out + r * os + (long)h * E + n) =
          uint2{cvt_pk_bf16(acc[0] * f, acc[1] * f),
                cvt_pk_bf16(acc[2] * f, acc[3] * f)};
    n0 += gridDim.z * NW * 16;
    if (n0 < E) weights();
  }
}

// ---- expanded attention, matrix cores -------------------------------------
// 128 query rows of one head a workgroup, 32 a wave; kv rows come in steps
// of 64.  kn [n, H*D] unrotated keys, lat [n, rank + rot] with the rotated
// part, vt [H*E, n] values transposed.  Row r of sequence s is the token at
// position first[s] + r - start[s]; start is a multiple of 8.
constexpr int KV = 64;
constexpr int VS = KV + 8;
constexpr int QT = 128;

constexpr int prefill_lds(int DP, int EP) {
  return (KV * (DP + 8) + EP * VS) * 2;
}

template <int DP, int EP>
__global__ __launch_bounds__(256, EP <= 128 ? 2 : 1)
void latent_attn_prefill_kernel(
    bf16* __restrict__ out, const bf16* __restrict__ q,
    const bf16* __restrict__ kn, const bf16* __restrict__ lat,
    const bf16* __restrict__ vt, const long* __restrict__ positions,
    const int* __restrict__ seq_start, const int* __restrict__ kv_start,
    const int* __restrict__ kv_first, const int* __restrict__ tiles,
    const float* __restrict__ sink, int H, int D, int E, int rank, int rot,
    long nkv, int window, float scale2, long qs, long os, Gate<bf16> gate) {
  constexpr int KS = DP + 8;                     // K row in LDS
  constexpr int KC = DP / 16, ET = EP / 32;
  constexpr int KLOADS = KV * DP / 8 / 256;      // 16-byte units a thread
  constexpr int VLOADS = KV * EP / 8 / 256;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  short* k_lds = reinterpret_cast<short*>(smem);
  short* v_lds = k_lds + KV * KS;

  // later rows see more: they start first; a head stays on one die
  const int tile = gridDim.y - 1 - blockIdx.y;
  const int s = tiles[2 * tile];
  const int t0 = seq_start[s] + tiles[2 * tile + 1];
  const int n = min(QT, seq_start[s + 1] - t0);
  if (n <= 0) return;
  const int h = blockIdx.x;
  const long kv0r = kv_start[s];                 // first kv row
  // positions relative to the first kv row's token
  const int p0 = (int)positions[t0] - kv_first[s];
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int col = lane & 31, hf = lane >> 5;
  const int row = wid * 32 + col;                // this lane's query row
  const int qp = p0 + row;

  short8_t qf[KC];
  {
    const bf16* qr = q + (long)(t0 + row) * qs + (long)h * (D + rot);
    #pragma unroll
    for (int c = 0; c < KC; ++c) {
      const int d = c * 16 + hf * 8;
      qf[c] = row < n && d < D + rot
          ? *reinterpret_cast<const short8_t*>(qr + d) : short8_t{};
    }
  }
  f32x16_t acc[ET];
  #pragma unroll
  for (int e = 0; e < ET; ++e) acc[e] = f32x16_t(0.f);
  float m = -FLT_MAX, l = 0.f;
  if (sink) {                        // counted once: by half of the lanes
    m = sink[h] * LOG2E;
    l = hf == 0 ? 1.f : 0.f;
  }

  const int last = p0 + n - 1;
  const int lo = max(0, p0 - window + 1);
  // first and last position of this wave's rows, for skipping whole steps
  const int w_first = p0 + wid * 32, w_last = min(w_first + 31, last);

  uint4 kr[KLOADS], vr[VLOADS];
  auto fetch = [&](int kv) {
    #pragma unroll
    for (int i = 0; i < KLOADS; ++i) {
      const int u = tid + 256 * i;
      const int p = kv + u / (DP / 8), d = (u % (DP / 8)) * 8;
      kr[i] = uint4{0, 0, 0, 0};
      if (p <= last && d < D + rot)
        kr[i] = *reinterpret_cast<const uint4*>(
            d < D ? kn + (kv0r + p) * ((long)H * D) + (long)h * D + d
                  : lat + (kv0r + p) * (rank + rot) + rank + d - D);
    }
    #pragma unroll
    for (int i = 0; i < VLOADS; ++i) {
      const int u = tid + 256 * i;
      const int e = u / 8, p = kv + (u % 8) * 8;
      vr[i] = uint4{0, 0, 0, 0};
      if (e < E && p <= last)
        vr[i] = *reinterpret_cast<const uint4*>(
            vt + ((long)h * E + e) * nkv + kv0r + p);
    }
  };
  auto stage = [&]() {
    #pragma unroll
    for (int i = 0; i < KLOADS; ++i) {
      const int u = tid + 256 * i;
      *reinterpret_cast<uint4*>(k_lds + (u / (DP / 8)) * KS +
                                (u % (DP / 8)) * 8) = kr[i];
    }
    #pragma unroll
    for (int i = 0; i < VLOADS; ++i) {
      const int u = tid + 256 * i;
      *reinterpret_cast<uint4*>(v_lds + (u / 8) * VS + (u % 8) * 8) = vr[i];
    }
  };

  // matrix row i of a 32-token block takes this token's key, so that the
  // scores a lane holds are 8 consecutive tokens
  const int krow = (col & 16) + ((col >> 2) & 1) * 8 + ((col >> 3) & 1) * 4 +
                   (col & 3);
  const int kv_first_step = lo / KV * KV;
  fetch(kv_first_step);
  for (int kv = kv_first_step; kv <= last; kv += KV) {
    stage();
    __syncthreads();
    if (kv + KV <= last) fetch(kv + KV);
    const bool any = kv <= w_last && kv + KV - 1 > w_first - window &&
                     w_first <= last;
    if (any) {
      f32x16_t sc[2];
      #pragma unroll
      for (int b = 0; b < 2; ++b) {
        sc[b] = f32x16_t(0.f);
        #pragma unroll
        for (int c = 0; c < KC; ++c)
          sc[b] = mfma32(*reinterpret_cast<const short8_t*>(
                             k_lds + (b * 32 + krow) * KS + c * 16 + hf * 8),
                         qf[c], sc[b]);
      }
      // token of sc[b][r]: kv + b*32 + (r>>3)*16 + hf*8 + (r&7)
      const bool full = kv + KV - 1 <= w_first && kv > w_last - window;
      float mx = m;
      #pragma unroll
      for (int b = 0; b < 2; ++b)
        #pragma unroll
        for (int r = 0; r < 16; ++r) {
          float x = sc[b][r] * scale2;
          if (!full) {
            const int p = kv + b * 32 + (r >> 3) * 16 + hf * 8 + (r & 7);
            if (p > qp || p <= qp - window) x = -FLT_MAX;
          }
          sc[b][r] = x;
          mx = fmaxf(mx, x);
        }
      mx = fmaxf(mx, __shfl_xor(mx, 32));
      if (!__all(mx == m)) {
        const float alpha = m == -FLT_MAX ? 0.f : exp2_fast(m - mx);
        #pragma unroll
        for (int e = 0; e < ET; ++e)
          #pragma unroll
          for (int r = 0; r < 16; ++r) acc[e][r] *= alpha;
        l *= alpha;
        m = mx;
      }
      // a column without a visible key yet has m = -FLT_MAX: with base 0 its
      // masked scores weigh exp2(-FLT_MAX) = 0
      const float base = m == -FLT_MAX ? 0.f : m;
      short8_t ph[4], pl[4];
      #pragma unroll
      for (int b = 0; b < 2; ++b)
        #pragma unroll
        for (int c = 0; c < 2; ++c) {
          float p[8];
          #pragma unroll
          for (int j = 0; j < 8; ++j) {
            p[j] = exp2_fast(sc[b][c * 8 + j] - base);
            l += p[j];
          }
          split_bf16x8(p, &ph[b * 2 + c], &pl[b * 2 + c]);
        }
      #pragma unroll
      for (int e = 0; e < ET; ++e)
        #pragma unroll
        for (int c = 0; c < 4; ++c) {
          const short8_t vf = *reinterpret_cast<const short8_t*>(
              v_lds + (e * 32 + col) * VS + c * 16 + hf * 8);
          acc[e] = mfma32(vf, ph[c], acc[e]);
          acc[e] = mfma32(vf, pl[c], acc[e]);
        }
    }
    __syncthreads();
  }
  l += __shfl_xor(l, 32);
  if (row >= n) return;
  const float inv = gate(t0 + row, h) / l;
  bf16* orow = out + (long)(t0 + row) * os + (long)h * E;
  #pragma unroll
  for (int e = 0; e < ET; ++e)
    #pragma unroll
    for (int r = 0; r < 16; r += 4) {
      const int c = e * 32 + 8 * (r >> 2) + 4 * hf;
      if (c < E)
        *reinterpret_cast<uint2*>(orow + c) = uint2{
            cvt_pk_bf16(acc[e][r] * inv, acc[e][r + 1] * inv),
            cvt_pk_bf16(acc[e][r + 2] * inv, acc[e][r + 3] * inv)};
    }
}

template <typename K> void allow_lds(K kernel, int bytes) {
  if (bytes > 65536)
    HIP_CHECK(hipFuncSetAttribute(
        reinterpret_cast<const void*>(kernel),
        hipFuncAttributeMaxDynamicSharedMemorySize, bytes));
}

}  // namespace

bool latent_sizes_fit(int D, int E, int rank, int rot) {
  return D % 8 == 0 && E % 8 == 0 && rank % 8 == 0 && rot % 8 == 0 &&
         D + rot <= 256 && E <= 256 && rank <= 512 && rot <= 64;
}

template <typename T>
void launch_latent_rope_append(T* q, const T* kv, const float* w,
                               const long* positions, const double* freqs,
                               const long* slot_mapping, T* cache, long rows,
                               int H, int D, int rank, int rot, long qs,
                               long ks, float eps, float gain,
                               const SideRelu<T>& side, hipStream_t stream) {
  if (rows == 0 || (rot == 0 && !kv && !side.n)) return;
  const dim3 grid((unsigned)rows, 1 + side_blocks(side.n));
  const size_t lds = (rot + 2) * sizeof(float);
  auto aligned = [](const T* p) {
    return reinterpret_cast<uintptr_t>(p) % (4 * sizeof(T)) == 0;
  };
  const bool vec = rank % 4 == 0 && rot % 4 == 0 && D % 4 == 0 &&
                   qs % 4 == 0 && ks % 4 == 0 && aligned(q) && aligned(kv);
  if (vec)
    latent_rope_append_kernel<T, 4><<<grid, 256, lds, stream>>>(
        q, kv, w, positions, freqs, slot_mapping, cache, H, D, rank, rot, qs,
        ks, eps, gain, side);
  else
    latent_rope_append_kernel<T, 1><<<grid, 256, lds, stream>>>(
        q, kv, w, positions, freqs, slot_mapping, cache, H, D, rank, rot, qs,
        ks, eps, gain, side);
}

void launch_latent_gather(bf16* out, const bf16* cache, const long* slots,
                          long rows, int width, hipStream_t stream) {
  if (rows == 0) return;
  const long total = rows * (width / 8);
  latent_gather_kernel<<<(unsigned)((total + 255) / 256), 256, 0, stream>>>(
      reinterpret_cast<uint4*>(out), reinterpret_cast<const uint4*>(cache),
      slots, total, width / 8);
}

// `fast`: bf16, N and K multiples of 8, 16-byte aligned rows
template <typename T>
void launch_head_gemm(T* out, const T* x, const T* w, const int* rows_in,
                      const int* rows_out, long R, int H, int N, int K,
                      long xr, long xh, long wn, long wh, long outr,
                      long outh, const T* g, long gs, bool fast,
                      hipStream_t stream) {
  if (R == 0) return;
  const Gate<T> gate{g, gs};
  const HeadGemm a{rows_in, rows_out, R, N, K, xr, xh, wn, wh, outr, outh};
  if constexpr (sizeof(T) == 2) {
    if (fast) {
      const unsigned nx = (unsigned)((N + 63) / 64);
      #define RUN(CT)                                                       \
        head_gemm_kernel<CT>                                                \
            <<<dim3(nx, (unsigned)((R + 16 * CT - 1) / (16 * CT)),          \
                    (unsigned)H), 256, 0, stream>>>(out, x, w, a, gate)
      if (R <= 16) RUN(1);
      else RUN(2);
      #undef RUN
      return;
    }
  }
  head_gemm_general_kernel<T>
      <<<dim3((unsigned)R, (unsigned)H), 256, 0, stream>>>(out, x, w, a,
                                                           gate);
}

template <typename T>
void launch_latent_attn_general(T* out, const T* qa, const T* q,
                                const T* cache, const int* block_tables,
                                const long* positions, const int* rows,
                                const int* row_seq, const float* sink,
                                long R, int max_blocks, int H, int D,
                                int rank, int rot, int window, float scale,
                                long qs, hipStream_t stream) {
  if (R == 0) return;
  if (rank > 256 * MAX_RPT || rot > 4096)
    throw std::runtime_error("latent_attn_general: latent size");
  latent_attn_general_kernel<T>
      <<<dim3((unsigned)R, (unsigned)H), 256,
         (rank + rot + TILE) * sizeof(float), stream>>>(
          out, qa, q, cache, block_tables, positions, rows, row_seq, sink,
          max_blocks, H, D, rank, rot, window, scale, qs);
}

void launch_latent_attn_decode(bf16* out, float* partial, const bf16* qa,
                               const bf16* q, const bf16* cache,
                               const int* block_tables, const long* positions,
                               const int* rows, const int* row_seq,
                               const float* sink, long R, int max_blocks,
                               int H, int D, int rank, int rot, int window,
                               float scale, long qs, int split,
                               hipStream_t stream) {
  if (R == 0) return;
  #define RUN(RP, XP, HT, EXACT)                                            \
    {                                                                       \
      allow_lds(&latent_attn_decode_kernel<RP, XP, HT, EXACT>,              \
                decode_lds(RP, XP));                                        \
      latent_attn_decode_kernel<RP, XP, HT, EXACT>                          \
          <<<dim3((unsigned)R, (unsigned)((H + 16 * HT - 1) / (16 * HT)),   \
                  (unsigned)split), 256, decode_lds(RP, XP), stream>>>(     \
              out, partial, qa, q, cache, block_tables, positions, rows,    \
              row_seq, sink, max_blocks, H, D, rank, rot, window,           \
              scale * LOG2E, qs);                                           \
      done = true;                                                          \
    }
  #define CASE(RP, XP)                                                      \
    if (!done && rank <= RP && rot <= XP) {                                 \
      if (H <= 16) RUN(RP, XP, 1, false) else RUN(RP, XP, 2, false)         \
    }
  bool done = false;
  if (rank == 512 && rot == 64) {
    if (H <= 16) RUN(512, 64, 1, true) else RUN(512, 64, 2, true)
  }
  CASE(64, 32) CASE(64, 64) CASE(128, 32) CASE(128, 64) CASE(256, 32)
  CASE(256, 64) CASE(512, 32) CASE(512, 64)
  #undef CASE
  #undef RUN
  if (!done) throw std::runtime_error("latent_attn_decode: latent size");
}

void launch_latent_merge_values(bf16* out, const float* partial,
                                const bf16* uv, const int* rows, long R,
                                int split, int H, int E, int rank, long os,
                                const bf16* g, long gs, hipStream_t stream) {
  if (R == 0) return;
  // few rows: fewer a workgroup, then fewer values a workgroup
  int rb = 16;
  while (rb > 1 && (R + rb - 1) / rb * H < 256) rb /= 2;
  const long units = R * H;
  const bool wide = units >= 128 && units <= 4096;
  const unsigned nz = units < 128 ? (unsigned)((E + 63) / 64) : 1;
  const dim3 grid((unsigned)((R + rb - 1) / rb), (unsigned)H, nz);
  auto run = [&](auto kernel, int threads) {
    kernel<<<grid, threads, 16 * (rank + 8) * 2, stream>>>(
        out, partial, uv, rows, R, split, H, E, rank, os, Gate<bf16>{g, gs});
  };
  #define CASE(RB)                                                          \
    if (rb == RB)                                                           \
      wide ? run(&latent_merge_values_kernel<RB, 8>, 512)                   \
           : run(&latent_merge_values_kernel<RB, 4>, 256);
  CASE(1) CASE(2) CASE(4) CASE(8) CASE(16)
  #undef CASE
}

void launch_latent_attn_prefill(bf16* out, const bf16* q, const bf16* kn,
                                const bf16* lat, const bf16* vt,
                                const long* positions, const int* seq_start,
                                const int* kv_start, const int* kv_first,
                                const int* tiles, const float* sink,
                                int num_tiles, int H, int D, int E, int rank,
                                int rot, long nkv, int window, float scale,
                                long qs, long os, const bf16* g, long gs,
                                hipStream_t stream) {
  if (num_tiles == 0) return;
  #define CASE(DP, EP)                                                      \
    if (D + rot <= DP && E <= EP) {                                         \
      allow_lds(&latent_attn_prefill_kernel<DP, EP>, prefill_lds(DP, EP));  \
      latent_attn_prefill_kernel<DP, EP>                                    \
          <<<dim3((unsigned)H, (unsigned)num_tiles), 256,                   \
             prefill_lds(DP, EP), stream>>>(                                \
              out, q, kn, lat, vt, positions, seq_start, kv_start,          \
              kv_first, tiles, sink, H, D, E, rank, rot, nkv, window,       \
              scale * LOG2E, qs, os, Gate<bf16>{g, gs});                    \
      return;                                                               \
    }
  CASE(64, 64) CASE(96, 64) CASE(64, 128) CASE(96, 128) CASE(128, 128)
  CASE(192, 128) CASE(256, 128) CASE(128, 256) CASE(192, 256) CASE(256, 256)
  #undef CASE
  throw std::runtime_error("latent_attn_prefill: head sizes");
}

#define INSTANTIATE(T)                                                      \
  template void launch_latent_rope_append<T>(                               \
      T*, const T*, const float*, const long*, const double*, const long*,  \
      T*, long, int, int, int, int, long, long, float, float,               \
      const SideRelu<T>&, hipStream_t);                                     \
  template void launch_head_gemm<T>(                                        \
      T*, const T*, const T*, const int*, const int*, long, int, int, int,  \
      long, long, long, long, long, long, const T*, long, bool,             \
      hipStream_t);                                                         \
  template void launch_latent_attn_general<T>(                              \
      T*, const T*, const T*, const T*, const int*, const long*,            \
      const int*, const int*, const float*, long, int, int, int, int, int,  \
      int, float, long, hipStream_t);
INSTANTIATE(bf16)
INSTANTIATE(float)
#undef INSTANTIATE
