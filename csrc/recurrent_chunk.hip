// Chunked prefill of the linear recurrences (gfx950 matrix cores, bf16 in,
// float state).  See csrc/recurrent.hip for the recurrences themselves.
//
// A prompt portion is cut into tiles of 64 tokens.  Within a tile, with
// b_t the running sum of log decays (a vector for gated linear attention, the
// scalar F_t for the matrix LSTM):
//
//   o_t   = (q_t exp(b_t)) S_in + sum_{s<=t} [q_t exp(b_t - b_s) . k_s] v_s
//   S_out = exp(b_C) S_in + sum_s (k_s exp(b_C - b_s)) v_s^T
//
// Lightning attention is the scalar case with b_t = (t + 1) log(decay).
//
// The matrix LSTM adds the input gate i_s to the exponents and keeps every
// sum divided by exp(m_t), m_t = F_t + max(m_in, max_{s<=t}(i_s - F_s)).
//
// Four passes: gates (running sums per tile), chunk_state (each tile's own
// contribution U, all tiles at once), chunk_scan (element-wise over the tiles
// of a sequence, U becomes the state S_in a tile starts from), chunk_out
// (outputs, per-head RMS norm and output gate, all tiles at once).
//
// Every exponent is <= 0: terms from an earlier 16-token block are taken
// relative to the decay at the start of the query's block, terms of the same
// block directly in float.  Float operands (states, decayed q and k, weights)
// enter the matrix cores as a bf16 high and low part, so the products keep
// ~16 bits; q, k, v themselves are bf16 already.
#include <float.h>

#include "common.h"
#include "recurrent.h"

namespace {

constexpr int C = 64;               // tokens per tile
constexpr int TS = C + 8;           // row of a token-minor LDS tile

DEV int pad32(int x) { return (x + 31) & ~31; }

struct Tile {
  int seq, first, t0, n, last;      // last: the sequence's final tile
};

DEV Tile load_tile(const int* tiles, const int* seq_start, int i) {
  Tile t;
  t.seq = tiles[2 * i];
  t.first = tiles[2 * i + 1];
  t.t0 = seq_start[t.seq] + t.first;
  const int left = seq_start[t.seq + 1] - t.t0;
  t.n = min(C, left);
  t.last = left <= C;
  return t;
}

// log of a constant decay; a decay of zero becomes one that vanishes in float
DEV float log_decay_of(float decay) { return logf(fmaxf(decay, 1e-38f)); }

DEV short8_t silu8(const short8_t& v) {
  union { unsigned u[4]; short8_t v; } r;
  #pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float a = bf16x8_at(v, 2 * i), b = bf16x8_at(v, 2 * i + 1);
    r.u[i] = cvt_pk_bf16(a / (1.f + __expf(-a)), b / (1.f + __expf(-b)));
  }
  return r.v;
}

// Rows [t0, t0+n) of src (column offset included, row stride `stride`) into
// dst[column][token], columns padded to `cols_pad` and tokens to C with zeros.
// ACT applies SiLU; f(token, column, 8 values in place) then transforms each
// 8-column chunk.
template <bool ACT, typename F>
DEV void stage_transposed(short* dst, short* dst_lo, const bf16* src,
                          long stride, int n, int cols, int cols_pad, F f) {
  const int units = 32 * (cols_pad / 8);
  for (int u = threadIdx.x; u < units; u += 256) {
    const int p = u & 31, c = (u >> 5) * 8;
    short8_t hi[2], lo[2];
    #pragma unroll
    for (int k = 0; k < 2; ++k) {
      const int s = 2 * p + k;
      hi[k] = short8_t{};
      lo[k] = short8_t{};
      if (s < n && c < cols) {
        hi[k] = *reinterpret_cast<const short8_t*>(src + s * stride + c);
        if constexpr (ACT) hi[k] = silu8(hi[k]);
        if (dst_lo) {
          float x[8];
          #pragma unroll
          for (int i = 0; i < 8; ++i) x[i] = bf16x8_at(hi[k], i);
          f(s, c, x);
          split_bf16x8(x, &hi[k], &lo[k]);
        }
      }
    }
    #pragma unroll
    for (int i = 0; i < 8; ++i) {
      *reinterpret_cast<unsigned*>(dst + (c + i) * TS + 2 * p) =
          (unsigned)(unsigned short)hi[0][i] |
          ((unsigned)(unsigned short)hi[1][i] << 16);
      if (dst_lo)
        *reinterpret_cast<unsigned*>(dst_lo + (c + i) * TS + 2 * p) =
            (unsigned)(unsigned short)lo[0][i] |
            ((unsigned)(unsigned short)lo[1][i] << 16);
    }
  }
}

// ---- gates ----------------------------------------------------------------

// b[t, c]: running sum within the tile of log_sigmoid(a2[c] . a1h_t + b)/tau
template <int RMAX>
__global__ __launch_bounds__(256) void gla_chunk_gates_kernel(
    float* __restrict__ b, const bf16* __restrict__ a1h,
    const bf16* __restrict__ a2, const float* __restrict__ a2b,
    const int* __restrict__ seq_start, const int* __restrict__ tiles,
    int channels, int rank, float inv_tau, long stride) {
  __shared__ float x[C][RMAX];
  const Tile t = load_tile(tiles, seq_start, blockIdx.x);
  if (t.n <= 0) return;
  for (int u = threadIdx.x; u < C * RMAX; u += 256) {
    const int s = u / RMAX, r = u % RMAX;
    x[s][r] = s < t.n && r < rank
        ? Elem<bf16>::ld(a1h + (t.t0 + s) * stride + r) : 0.f;
  }
  __syncthreads();
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= channels) return;
  float w[RMAX];
  #pragma unroll
  for (int r = 0; r < RMAX; ++r)
    w[r] = r < rank ? Elem<bf16>::ld(a2 + (long)c * rank + r) : 0.f;
  const float bias = a2b[c];
  float sum = 0.f;
  for (int s = 0; s < t.n; ++s) {
    float z = bias;
    #pragma unroll
    for (int r = 0; r < RMAX; ++r) z += w[r] * x[s][r];
    sum += log_sigmoid(z) * inv_tau;
    b[(long)(t.t0 + s) * channels + c] = sum;
  }
}

// gates[t, 0:H] = log input gate i, gates[t, H:2H] = running sum F;
// info[tile, h] = (F_C, max_s(F_C - F_s + i_s)).  One wave per (tile, head).
__global__ __launch_bounds__(64) void mlstm_chunk_gates_kernel(
    float* __restrict__ gates, float* __restrict__ info,
    const float* __restrict__ raw, const float* __restrict__ ib,
    const float* __restrict__ fb, const int* __restrict__ seq_start,
    const int* __restrict__ tiles, int H, float cap) {
  const Tile t = load_tile(tiles, seq_start, blockIdx.x);
  if (t.n <= 0) return;
  const int h = blockIdx.y, s = threadIdx.x;
  const bool in = s < t.n;
  const long at = (long)(t.t0 + s) * 2 * H + h;
  float i = -FLT_MAX, f = 0.f;
  if (in) {
    i = cap * tanhf((raw[at] + ib[h]) / cap);
    f = log_sigmoid(cap * tanhf((raw[at + H] + fb[h]) / cap));
  }
  #pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const float v = __shfl_up(f, o);
    if (s >= o) f += v;
  }
  if (in) {
    gates[at] = i;
    gates[at + H] = f;
  }
  const float total = __shfl(f, t.n - 1);
  const float m = wave_reduce_max(in ? total - f + i : -FLT_MAX);
  if (s == 0) {
    info[((long)blockIdx.x * H + h) * 2] = total;
    info[((long)blockIdx.x * H + h) * 2 + 1] = m;
  }
}

// ---- a tile's own state contribution --------------------------------------
// U[tile, h, e, d] (transposed state) and, for the matrix LSTM, nU[tile, h, d]
template <Kind K>
__global__ __launch_bounds__(256) void chunk_state_kernel(
    float* __restrict__ U, float* __restrict__ nU, const bf16* __restrict__ k,
    const bf16* __restrict__ v, const float* __restrict__ gates,
    const float* __restrict__ info, const int* __restrict__ seq_start,
    const int* __restrict__ tiles, int H, int D, int E, long stride) {
  extern __shared__ __attribute__((aligned(16))) char sm[];
  const int DP = pad32(D), EP = pad32(E);
  short* kt = reinterpret_cast<short*>(sm);      // [DP][TS]
  short* kt_lo = kt + DP * TS;
  short* vt = kt_lo + DP * TS;                   // [EP][TS]
  const Tile t = load_tile(tiles, seq_start, blockIdx.x);
  if (t.n <= 0) return;
  const int h = blockIdx.y;
  const long th = (long)blockIdx.x * H + h;

  const float* bh = gates + ((long)t.t0 * H + h) * D;     // GLA: [s][H*D]
  const float* gh = gates + (long)t.t0 * 2 * H + h;       // mLSTM: i, F
  float fc = 0.f, mu = 0.f;
  if constexpr (K == MLSTM) { fc = info[2 * th]; mu = info[2 * th + 1]; }
  if constexpr (K == LIGHTNING) fc = log_decay_of(gates[h]);
  stage_transposed<K == LIGHTNING>(
      kt, kt_lo, k + (long)t.t0 * stride + (long)h * D, stride, t.n, D, DP,
      [&](int s, int c, float* x) {
        if constexpr (K == MLSTM) {
          const float w = __expf(fc - gh[s * 2 * H + H] + gh[s * 2 * H] - mu);
          #pragma unroll
          for (int i = 0; i < 8; ++i) x[i] *= w;
        } else if constexpr (K == LIGHTNING) {
          const float w = __expf(fc * (t.n - 1 - s));
          #pragma unroll
          for (int i = 0; i < 8; ++i) x[i] *= w;
        } else {
          const float* bs = bh + (long)s * H * D + c;
          const float* bc = bh + (long)(t.n - 1) * H * D + c;
          #pragma unroll
          for (int i = 0; i < 8; ++i) x[i] *= __expf(bc[i] - bs[i]);
        }
      });
  stage_transposed<K == LIGHTNING>(vt, nullptr, v + (long)t.t0 * stride + (long)h * E, stride,
                   t.n, E, EP, [](int, int, float*) {});
  __syncthreads();

  if constexpr (K == MLSTM) {
    for (int d = threadIdx.x; d < D; d += 256) {
      float s = 0.f;
      for (int i = 0; i < C; i += 8) {
        const short8_t a = *reinterpret_cast<short8_t*>(kt + d * TS + i);
        const short8_t b = *reinterpret_cast<short8_t*>(kt_lo + d * TS + i);
        #pragma unroll
        for (int j = 0; j < 8; ++j) s += bf16x8_at(a, j) + bf16x8_at(b, j);
      }
      nU[th * D + d] = s;
    }
  }
  const int lane = threadIdx.x & 63, col = lane & 31, hf = lane >> 5;
  const int nd = DP / 32, ne = EP / 32;
  for (int u = threadIdx.x >> 6; u < nd * ne; u += 4) {
    const int et = u / nd, dt = u % nd;
    f32x16_t acc = f32x16_t(0.f);
    #pragma unroll
    for (int c = 0; c < C / 16; ++c) {
      const int at = c * 16 + hf * 8;
      const short8_t a = *reinterpret_cast<short8_t*>(
          vt + (et * 32 + col) * TS + at);
      acc = mfma32(a, *reinterpret_cast<short8_t*>(
                          kt + (dt * 32 + col) * TS + at), acc);
      acc = mfma32(a, *reinterpret_cast<short8_t*>(
                          kt_lo + (dt * 32 + col) * TS + at), acc);
    }
    const int d = dt * 32 + col;
    if (d < D) {
      #pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int e = et * 32 + (r & 3) + 8 * (r >> 2) + 4 * hf;
        if (e < E) U[(th * E + e) * D + d] = acc[r];
      }
    }
  }
}

// ---- over the tiles of a sequence -----------------------------------------
// U[tile] becomes the state the tile starts from; the state after the last
// tile goes to the pool.  A thread owns four neighbouring d of one e; the
// matrix LSTM's extra block (blockIdx.x == gridDim.x - 1) carries n and m_in.
template <Kind K>
__global__ __launch_bounds__(256) void chunk_scan_kernel(
    float* __restrict__ U, float* __restrict__ nU, float* __restrict__ m_in,
    float* __restrict__ S, float* __restrict__ n_pool,
    const float* __restrict__ m_pool, const float* __restrict__ gates,
    const float* __restrict__ info, const int* __restrict__ seq_start,
    const long* __restrict__ positions, const int* __restrict__ slots,
    const int* __restrict__ tile_start, int H, int D, int E) {
  const int s = blockIdx.z, h = blockIdx.y;
  const int t0 = seq_start[s], t1 = seq_start[s + 1];
  const int c0 = tile_start[s];
  // a padded tile list may reach past the real tokens
  const int c1 = min(tile_start[s + 1], c0 + (t1 - t0 + C - 1) / C);
  if (t1 <= t0 || c1 <= c0) return;
  const int slot = slots[s];
  const bool fresh = slot < 0 || positions[t0] == 0;
  const bool nblock = K == MLSTM && blockIdx.x == gridDim.x - 1;
  const int u = (nblock ? 0 : blockIdx.x * 1024) + threadIdx.x * 4;
  const int size = nblock ? D : D * E;
  if (u >= size) return;
  const int e = u / D, d = u % D;
  const long step = (long)H * size;
  float* p = (nblock ? nU : U) + ((long)c0 * H + h) * size + u;
  // pool element i: S is kept [D][E]
  float* pool = nblock ? n_pool + ((long)max(slot, 0) * H + h) * D + d
                       : S + ((long)max(slot, 0) * H + h) * D * E +
                             (long)d * E + e;
  const int pstep = nblock ? 1 : E;
  float st[4];
  #pragma unroll
  for (int i = 0; i < 4; ++i) st[i] = fresh ? 0.f : pool[i * pstep];
  float m = 0.f;
  if (K == MLSTM && !fresh) m = m_pool[(long)slot * H + h];

  constexpr int AHEAD = 4;
  for (int c = c0; c < c1; c += AHEAD) {
    float4 x[AHEAD], a[AHEAD];
    #pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      if (c + j >= c1) break;
      x[j] = *reinterpret_cast<float4*>(p + j * step);
      if constexpr (K == MLSTM) {
        const float* f = info + ((long)(c + j) * H + h) * 2;
        a[j].x = f[0];
        a[j].y = f[1];
      } else if constexpr (K == LIGHTNING) {
        const int n = min(t1 - t0 - (c + j - c0) * C, C);
        a[j].x = log_decay_of(gates[h]) * n;
      } else {
        // the last token of the tile carries the tile's whole decay
        const int row = min(t0 + (c + j - c0 + 1) * C, t1) - 1;
        a[j] = *reinterpret_cast<const float4*>(
            gates + ((long)row * H + h) * D + d);
      }
    }
    #pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      if (c + j >= c1) break;
      *reinterpret_cast<float4*>(p + j * step) =
          make_float4(st[0], st[1], st[2], st[3]);
      if constexpr (K == MLSTM) {
        if (nblock && threadIdx.x == 0) m_in[(long)(c + j) * H + h] = m;
        const float mn = fmaxf(a[j].x + m, a[j].y);
        const float fs = expf(a[j].x + m - mn), us = expf(a[j].y - mn);
        m = mn;
        st[0] = st[0] * fs + x[j].x * us;
        st[1] = st[1] * fs + x[j].y * us;
        st[2] = st[2] * fs + x[j].z * us;
        st[3] = st[3] * fs + x[j].w * us;
      } else if constexpr (K == LIGHTNING) {
        const float f = expf(a[j].x);
        st[0] = st[0] * f + x[j].x;
        st[1] = st[1] * f + x[j].y;
        st[2] = st[2] * f + x[j].z;
        st[3] = st[3] * f + x[j].w;
      } else {
        st[0] = st[0] * expf(a[j].x) + x[j].x;
        st[1] = st[1] * expf(a[j].y) + x[j].y;
        st[2] = st[2] * expf(a[j].z) + x[j].z;
        st[3] = st[3] * expf(a[j].w) + x[j].w;
      }
    }
    p += AHEAD * step;
  }
  if (slot < 0) return;
  #pragma unroll
  for (int i = 0; i < 4; ++i) pool[i * pstep] = st[i];
}

// ---- outputs ----------------------------------------------------------------
// ET: 32-column blocks of the value size per wave (E <= 128 * ET)
template <int ET, Kind K>
__global__ __launch_bounds__(256) void chunk_out_kernel(
    bf16* __restrict__ y, float* __restrict__ o_raw,
    const float* __restrict__ S, const float* __restrict__ n_in, const float* __restrict__ m_in,
    float* __restrict__ m_pool, const bf16* __restrict__ q,
    const bf16* __restrict__ k, const bf16* __restrict__ v,
    const bf16* __restrict__ g, const float* __restrict__ gates,
    const float* __restrict__ w, const int* __restrict__ seq_start,
    const int* __restrict__ tiles, const int* __restrict__ slots, int H,
    int D, int E, long stride, float qscale, float eps) {
  extern __shared__ __attribute__((aligned(16))) char sm[];
  const int DP = pad32(D), EP = pad32(E), DS = DP + 8, BS = DP + 4;
  short* q_lds = reinterpret_cast<short*>(sm);   // [C][DS]
  short* k_lds = q_lds + C * DS;                 // [C][DS]
  short* vt = k_lds + C * DS;                    // [EP][TS]
  short* a_hi = vt + EP * TS;                    // [C][TS] weights (t, s)
  short* a_lo = a_hi + C * TS;
  float* red = reinterpret_cast<float*>(a_lo + C * TS);   // [4][C]
  float* tf = red + 4 * C;                       // mLSTM: F_t
  float* ti = tf + C;                            //        i_t
  float* tm = ti + C;                            //        m_t
  float* tden = tm + C;                          //        own-tile n . q
  float* tinv = tden + C;                        //        1 / denominator
  float* b_lds = tinv + C;                       // GLA: [C][BS]

  const Tile t = load_tile(tiles, seq_start, blockIdx.x);
  if (t.n <= 0) return;
  const int h = blockIdx.y;
  const long th = (long)blockIdx.x * H + h;
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;

  // ---- stage ----
  for (int u = tid; u < C * (DP / 8); u += 256) {
    const int s = u / (DP / 8), c = (u % (DP / 8)) * 8;
    short8_t a{}, b{};
    if (s < t.n && c < D) {
      const long at = (long)(t.t0 + s) * stride + (long)h * D + c;
      a = *reinterpret_cast<const short8_t*>(q + at);
      b = *reinterpret_cast<const short8_t*>(k + at);
      if constexpr (K == LIGHTNING) { a = silu8(a); b = silu8(b); }
    }
    *reinterpret_cast<short8_t*>(q_lds + s * DS + c) = a;
    *reinterpret_cast<short8_t*>(k_lds + s * DS + c) = b;
    if constexpr (K == GLA) {
      // rows past the end repeat the last one: every exponent stays finite
      const float* src = gates +
          ((long)(t.t0 + min(s, t.n - 1)) * H + h) * D + c;
      float4 x{0.f, 0.f, 0.f, 0.f}, z = x;
      if (c < D) {
        x = *reinterpret_cast<const float4*>(src);
        z = *reinterpret_cast<const float4*>(src + 4);
      }
      *reinterpret_cast<float4*>(b_lds + s * BS + c) = x;
      *reinterpret_cast<float4*>(b_lds + s * BS + c + 4) = z;
    }
  }
  stage_transposed<K == LIGHTNING>(vt, nullptr, v + (long)t.t0 * stride + (long)h * E, stride,
                   t.n, E, EP, [](int, int, float*) {});
  float mi = 0.f, ld = 0.f;
  if constexpr (K == LIGHTNING) ld = log_decay_of(gates[h]);
  if constexpr (K == MLSTM) {
    mi = m_in[th];
    if (wid == 0) {
      const int s = min(lane, t.n - 1);
      const long at = (long)(t.t0 + s) * 2 * H + h;
      const float i = gates[at], f = gates[at + H];
      float x = i - f;
      #pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const float r = __shfl_up(x, o);
        if (lane >= o) x = fmaxf(x, r);
      }
      tf[lane] = f;
      ti[lane] = i;
      tm[lane] = f + fmaxf(mi, x);
      if (t.last && lane == t.n - 1 && slots[t.seq] >= 0)
        m_pool[(long)slots[t.seq] * H + h] = tm[lane];
    }
  }
  __syncthreads();

  // ---- weights of the tile's own tokens: wave = 16 query rows ----
  {
    const int cl = lane & 15, gr = lane >> 4;
    const int r0 = wid * 16 + gr * 4;            // rows r0..r0+3, this lane
    const float* ref = b_lds + (wid * 16 - 1) * BS;
    float den[4] = {0.f, 0.f, 0.f, 0.f};
    for (int J = 0; J < 4; ++J) {
      const int s = J * 16 + cl;
      float a[4] = {0.f, 0.f, 0.f, 0.f};
      if (J < wid || (K != GLA && J == wid)) {
        f32x4_t acc = f32x4_t(0.f);
        for (int c = 0; c < DP; c += 32) {
          const int d = c + gr * 8;
          const short8_t qv = *reinterpret_cast<short8_t*>(
              q_lds + (wid * 16 + cl) * DS + d);
          const short8_t kv = *reinterpret_cast<short8_t*>(
              k_lds + s * DS + d);
          if constexpr (K != GLA) {
            acc = mfma16(qv, kv, acc);
          } else {
            const float* bq = b_lds + (wid * 16 + cl) * BS + d;
            const float* bk = b_lds + s * BS + d;
            float x[8], z[8];
            #pragma unroll
            for (int i = 0; i < 8; ++i) {
              const float rf = ref[d + i];
              x[i] = bf16x8_at(qv, i) * __expf(bq[i] - rf);
              z[i] = bf16x8_at(kv, i) * __expf(rf - bk[i]);
            }
            short8_t xh, xl, zh, zl;
            split_bf16x8(x, &xh, &xl);
            split_bf16x8(z, &zh, &zl);
            acc = mfma16(xh, zh, acc);
            acc = mfma16(xh, zl, acc);
            acc = mfma16(xl, zh, acc);
          }
        }
        #pragma unroll
        for (int r = 0; r < 4; ++r) a[r] = acc[r];
      } else if (J == wid) {
        // same block: every pair directly, in float
        for (int d = 0; d < D; d += 4) {
          const float4 kv = Elem<bf16>::ld4(
              reinterpret_cast<bf16*>(k_lds + s * DS + d));
          const float4 bk = *reinterpret_cast<float4*>(b_lds + s * BS + d);
          #pragma unroll
          for (int r = 0; r < 4; ++r) {
            const float4 qv = Elem<bf16>::ld4(
                reinterpret_cast<bf16*>(q_lds + (r0 + r) * DS + d));
            const float4 bq = *reinterpret_cast<float4*>(
                b_lds + (r0 + r) * BS + d);
            // the minimum only matters for s > t, which is dropped below
            a[r] += qv.x * kv.x * __expf(fminf(bq.x - bk.x, 0.f)) +
                    qv.y * kv.y * __expf(fminf(bq.y - bk.y, 0.f)) +
                    qv.z * kv.z * __expf(fminf(bq.z - bk.z, 0.f)) +
                    qv.w * kv.w * __expf(fminf(bq.w - bk.w, 0.f));
          }
        }
      }
      #pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = r0 + r;
        float x = 0.f;
        if (s <= row) {
          x = a[r] * qscale;
          if constexpr (K == LIGHTNING) x *= __expf(ld * (row - s));
          if constexpr (K == MLSTM) {
            x *= __expf(tf[row] - tf[s] + ti[s] - tm[row]);
            den[r] += x;
          }
        }
        const unsigned short hi = f2bf(x);
        a_hi[row * TS + s] = (short)hi;
        a_lo[row * TS + s] = (short)f2bf(x - bf2f(hi));
      }
    }
    if constexpr (K == MLSTM) {
      #pragma unroll
      for (int r = 0; r < 4; ++r) {
        float x = den[r];
        #pragma unroll
        for (int o = 1; o < 16; o <<= 1) x += __shfl_xor(x, o);
        if (cl == 0) tden[r0 + r] = x;
      }
    }
  }
  __syncthreads();
  if constexpr (K == MLSTM) {
    // four threads a row finish the denominator with the incoming n
    const int row = tid >> 2, part = tid & 3;
    float x = 0.f;
    for (int d = part; d < D; d += 4)
      x += bf2f((unsigned short)q_lds[row * DS + d]) * n_in[th * D + d];
    x += __shfl_xor(x, 1);
    x += __shfl_xor(x, 2);
    if (part == 0) {
      x = x * qscale * __expf(tf[row] + mi - tm[row]) + tden[row];
      tinv[row] = 1.f / (fmaxf(fabsf(x), __expf(-tm[row])) + DEN_EPS);
    }
    __syncthreads();
  }

  // ---- O^T[e][t]: incoming state, then the tile's own tokens ----
  const int col = lane & 31, hf = lane >> 5;
  const int ne = EP / 32;
  f32x16_t acc[ET][2];
  #pragma unroll
  for (int i = 0; i < ET; ++i)
    #pragma unroll
    for (int tt = 0; tt < 2; ++tt) acc[i][tt] = f32x16_t(0.f);
  for (int c = 0; c < D; c += 16) {
    const int d = c + hf * 8;
    short8_t qh[2], ql[2];
    #pragma unroll
    for (int tt = 0; tt < 2; ++tt) {
      const int row = tt * 32 + col;
      qh[tt] = *reinterpret_cast<short8_t*>(q_lds + row * DS + d);
      if constexpr (K == GLA) {
        float x[8];
        #pragma unroll
        for (int i = 0; i < 8; ++i)
          x[i] = bf16x8_at(qh[tt], i) * __expf(b_lds[row * BS + d + i]);
        split_bf16x8(x, &qh[tt], &ql[tt]);
      }
    }
    #pragma unroll
    for (int i = 0; i < ET; ++i) {
      const int e = (wid + 4 * i) * 32 + col;
      if (wid + 4 * i >= ne) continue;
      float x[8] = {};
      if (e < E && d < D) {
        const float* sp = S + (th * E + e) * D + d;
        *reinterpret_cast<float4*>(x) = *reinterpret_cast<const float4*>(sp);
        *reinterpret_cast<float4*>(x + 4) =
            *reinterpret_cast<const float4*>(sp + 4);
      }
      short8_t sh, sl;
      split_bf16x8(x, &sh, &sl);
      #pragma unroll
      for (int tt = 0; tt < 2; ++tt) {
        acc[i][tt] = mfma32(sh, qh[tt], acc[i][tt]);
        acc[i][tt] = mfma32(sl, qh[tt], acc[i][tt]);
        if constexpr (K == GLA) acc[i][tt] = mfma32(sh, ql[tt], acc[i][tt]);
      }
    }
  }
  #pragma unroll
  for (int tt = 0; tt < 2; ++tt) {
    const int row = tt * 32 + col;
    float f = qscale;
    if constexpr (K == MLSTM) f *= __expf(tf[row] + mi - tm[row]);
    if constexpr (K == LIGHTNING) f *= __expf(ld * (row + 1));
    #pragma unroll
    for (int i = 0; i < ET; ++i)
      #pragma unroll
      for (int r = 0; r < 16; ++r) acc[i][tt][r] *= f;
    #pragma unroll
    for (int c = 0; c < 2 * (tt + 1); ++c) {
      const int at = c * 16 + hf * 8;
      const short8_t ah = *reinterpret_cast<short8_t*>(a_hi + row * TS + at);
      const short8_t al = *reinterpret_cast<short8_t*>(a_lo + row * TS + at);
      #pragma unroll
      for (int i = 0; i < ET; ++i) {
        if (wid + 4 * i >= ne) continue;
        const short8_t vf = *reinterpret_cast<short8_t*>(
            vt + ((wid + 4 * i) * 32 + col) * TS + at);
        acc[i][tt] = mfma32(vf, ah, acc[i][tt]);
        acc[i][tt] = mfma32(vf, al, acc[i][tt]);
      }
    }
    if constexpr (K == LIGHTNING) {
      if (row >= t.n) continue;
      #pragma unroll
      for (int i = 0; i < ET; ++i)
        #pragma unroll
        for (int r = 0; r < 16; r += 4) {
          const int e = (wid + 4 * i) * 32 + 8 * (r >> 2) + 4 * hf;
          if (e >= E) continue;
          *reinterpret_cast<float4*>(
              o_raw + ((long)(t.t0 + row) * H + h) * E + e) =
              make_float4(acc[i][tt][r], acc[i][tt][r + 1],
                          acc[i][tt][r + 2], acc[i][tt][r + 3]);
        }
      continue;
    }
    float ss = 0.f;
    #pragma unroll
    for (int i = 0; i < ET; ++i)
      #pragma unroll
      for (int r = 0; r < 16; ++r) {
        if constexpr (K == MLSTM) acc[i][tt][r] *= tinv[row];
        ss += acc[i][tt][r] * acc[i][tt][r];    // columns past E are zero
      }
    ss += __shfl_xor(ss, 32);
    if (hf == 0) red[wid * C + row] = ss;
  }
  if constexpr (K == LIGHTNING) return;
  __syncthreads();
  #pragma unroll
  for (int tt = 0; tt < 2; ++tt) {
    const int row = tt * 32 + col;
    if (row >= t.n) continue;
    const float ss = red[row] + red[C + row] + red[2 * C + row] +
                     red[3 * C + row];
    const float rs = 1.f / sqrtf(ss / E + eps);
    const bf16* gr = g + (long)(t.t0 + row) * stride + (long)h * E;
    bf16* yr = y + ((long)(t.t0 + row) * H + h) * E;
    #pragma unroll
    for (int i = 0; i < ET; ++i)
      #pragma unroll
      for (int r = 0; r < 16; r += 4) {
        const int e = (wid + 4 * i) * 32 + 8 * (r >> 2) + 4 * hf;
        if (e >= E) continue;
        const float4 wv = *reinterpret_cast<const float4*>(
            w + (K == MLSTM ? h * E : 0) + e);
        float gv[4];
        load_vec<bf16, 4>(gr + e, gv);
        float o[4];
        #pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float sg = 1.f / (1.f + __expf(-gv[j]));
          o[j] = acc[i][tt][r + j] * rs * (&wv.x)[j] *
                 (K == MLSTM ? sg : gv[j] * sg);
        }
        store_vec<bf16, 4>(yr + e, o);
      }
  }
}

constexpr size_t MAX_LDS = 160 * 1024;

size_t state_lds(int D, int E) {
  const int dp = (D + 31) / 32 * 32, ep = (E + 31) / 32 * 32;
  return (size_t)(2 * dp + ep) * TS * 2;
}

size_t out_lds(int D, int E, bool gla) {
  const int dp = (D + 31) / 32 * 32, ep = (E + 31) / 32 * 32;
  size_t n = (size_t)(2 * C * (dp + 8) + (ep + 2 * C) * TS) * 2;
  n += (4 + 5) * C * 4;
  if (gla) n += (size_t)C * (dp + 4) * 4;
  return n;
}

template <typename K> void allow_lds(K kernel, size_t bytes) {
  if (bytes > 65536)
    HIP_CHECK(hipFuncSetAttribute(
        reinterpret_cast<const void*>(kernel),
        hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes));
}

}  // namespace

bool recurrent_chunk_fits(int D, int E, int rank) {
  return D % 8 == 0 && E % 8 == 0 && E <= 256 && rank <= 64 &&
         state_lds(D, E) <= MAX_LDS && out_lds(D, E, true) <= MAX_LDS;
}

void launch_gla_chunk_gates(float* b, const bf16* a1h, const bf16* a2,
                            const float* a2b, const int* seq_start,
                            const int* tiles, int num_tiles, int channels,
                            int rank, float tau, long stride,
                            hipStream_t stream) {
  if (num_tiles == 0) return;
  const dim3 grid((unsigned)num_tiles, (unsigned)((channels + 255) / 256));
  #define GATES(R)                                                          \
    if (rank <= R) {                                                        \
      gla_chunk_gates_kernel<R><<<grid, 256, 0, stream>>>(                  \
          b, a1h, a2, a2b, seq_start, tiles, channels, rank, 1.f / tau,     \
          stride);                                                          \
      return;                                                               \
    }
  GATES(16) GATES(32) GATES(64)
  #undef GATES
  throw std::runtime_error("gla_chunk_gates: rank above 64");
}

void launch_mlstm_chunk_gates(float* gates, float* info, const float* raw,
                              const float* ib, const float* fb,
                              const int* seq_start, const int* tiles,
                              int num_tiles, int H, float cap,
                              hipStream_t stream) {
  if (num_tiles == 0) return;
  mlstm_chunk_gates_kernel<<<dim3((unsigned)num_tiles, (unsigned)H), 64, 0,
                             stream>>>(gates, info, raw, ib, fb, seq_start,
                                       tiles, H, cap);
}

template <Kind K>
static void run_chunk(bf16* y, float* o_raw, float* U, float* nU, float* m_in,
                      float* S, float* n_pool, float* m_pool, const bf16* q,
                      const bf16* k, const bf16* v, const bf16* g,
                      const float* gates, const float* info, const float* w,
                      const int* seq_start, const long* positions,
                      const int* slots, const int* tiles,
                      const int* tile_start, int num_tiles, int num_seqs,
                      int H, int D, int E, long stride, float qscale,
                      float eps, hipStream_t stream) {
  const dim3 grid((unsigned)num_tiles, (unsigned)H);
  const size_t l1 = state_lds(D, E), l2 = out_lds(D, E, K == GLA);
  allow_lds(&chunk_state_kernel<K>, l1);
  chunk_state_kernel<K><<<grid, 256, l1, stream>>>(
      U, nU, k, v, gates, info, seq_start, tiles, H, D, E, stride);
  const dim3 sgrid((unsigned)((D * E + 1023) / 1024 + (K == MLSTM ? 1 : 0)),
                   (unsigned)H, (unsigned)num_seqs);
  chunk_scan_kernel<K><<<sgrid, 256, 0, stream>>>(
      U, nU, m_in, S, n_pool, m_pool, gates, info, seq_start, positions,
      slots, tile_start, H, D, E);
  #define OUT(ET)                                                           \
    allow_lds(&chunk_out_kernel<ET, K>, l2);                                \
    chunk_out_kernel<ET, K><<<grid, 256, l2, stream>>>(                     \
        y, o_raw, U, nU, m_in, m_pool, q, k, v, g, gates, w, seq_start,     \
        tiles, slots, H, D, E, stride, qscale, eps)
  if (E <= 128) {
    OUT(1);
  } else {
    OUT(2);
  }
  #undef OUT
}

void launch_recurrent_chunk(Kind kind, bf16* y, float* o_raw, float* U,
                            float* nU, float* m_in, float* S, float* n_pool,
                            float* m_pool, const bf16* q, const bf16* k,
                            const bf16* v, const bf16* g, const float* gates,
                            const float* info, const float* w,
                            const int* seq_start, const long* positions,
                            const int* slots, const int* tiles,
                            const int* tile_start, int num_tiles,
                            int num_seqs, int H, int D, int E, long stride,
                            float qscale, float eps, hipStream_t stream) {
  if (num_tiles == 0 || num_seqs == 0) return;
  #define RUN(K)                                                            \
    if (kind == K)                                                          \
      run_chunk<K>(y, o_raw, U, nU, m_in, S, n_pool, m_pool, q, k, v, g,    \
                   gates, info, w, seq_start, positions, slots, tiles,      \
                   tile_start, num_tiles, num_seqs, H, D, E, stride,        \
                   qscale, eps, stream);
  RUN(GLA) RUN(MLSTM) RUN(LIGHTNING)
  #undef RUN
}
