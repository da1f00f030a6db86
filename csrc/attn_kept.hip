// Windowed softmax attention with kept first tokens over the paged cache
// (gfx950).
//
// Row t of position p sees the positions p - window < j <= p and j < keep of
// its sequence.  The softmax denominator of head h also has exp(sink[h]),
// once, without a value (null: nothing).  Values may be kept turned by their
// position; outputs are then turned back by the row's (rotary.h: neighbouring
// dimensions are a pair).
//
//   q       [T, H * D]  (token stride qs)    out [T, H * E] (token stride os)
//   k_cache [NB, G, 16, D]     v_cache [NB, G, E, 16]  (V^T per page)
//
// Three kernels:
//   general  any head sizes, bf16 or float, prefill and decode rows alike, one
//            workgroup per (row, head);
//   prefill  bf16 matrix cores, 64 query rows of one or two heads a workgroup;
//   decode   bf16 matrix cores, one row and up to 16 heads of a kv head a
//            workgroup, optionally split over the keys with a merge pass.
// The matrix-core kernels want D and E to be multiples of 8, at most 256;
// smaller sizes are padded with zeros in registers and LDS.
//
// Operand layouts (v_mfma_f32_32x32x16 / 16x16x32, bf16):  scores are formed
// transposed, S^T = K Q^T, with the K row that feeds matrix row i permuted so
// that the scores a lane holds are 8 consecutive tokens of one query column,
// which is the operand P^T of O^T = V^T P^T: weights never leave their
// registers, and V^T comes straight from the transposed pages.  The weights
// enter as a bf16 high and low part.  A pair of an output's dimensions is in
// one lane.
//
// BOUNDED: the caller knows that scores and sinks are small enough for their
// exponentials as they are (normed queries and keys: |score| <= D |scale|), so
// no running maximum is kept.
#include <float.h>

#include <type_traits>

#include "rotary.h"

#define PAGE 16

namespace {

constexpr float LOG2E = 1.4426950408889634f;
constexpr int TILE = 256;      // tokens per step of the general kernel
constexpr int MAX_EPT = 4;     // values per thread: E <= 1024

DEV float exp2_fast(float x) { return __builtin_amdgcn_exp2f(x); }

template <typename T> struct Kept {
  T* out;
  const T* q;
  const T* k_cache;
  const T* v_cache;
  const int* block_tables;
  const long* positions;
  const double* turn;        // [E / 2], null: values are not turned
  const float* sink;         // [H], null: none
  int max_blocks, H, G, D, E, window, keep;
  float scale;               // of the scores; times log2(e) where noted
  long qs, os;
};

// x[0], x[1] at columns c, c + 1 of an output at `pos` turned back
template <typename T>
DEV void turn_back(const Kept<T>& a, long pos, int c, float* x) {
  float cs[2];
  angle<T>(-pos, a.turn[c / 2], &cs[0], &cs[1]);
  turn_pairs<2>(x, cs);
}

template <typename T>
__global__ __launch_bounds__(256) void kept_attn_general_kernel(
    Kept<T> a, const int* __restrict__ row_seq) {
  extern __shared__ float smem[];
  float* q_lds = smem;                 // [D]
  float* p_lds = smem + a.D;           // [TILE]
  __shared__ float scratch[4];
  const long row = blockIdx.x;
  const int h = blockIdx.y, g = h / (a.H / a.G), tid = threadIdx.x;
  const int* bt = a.block_tables +
                  (long)(row_seq ? row_seq[row] : (int)row) * a.max_blocks;
  const long pos = a.positions[row];
  const long lo = pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;
  for (int i = tid; i < a.D; i += 256)
    q_lds[i] = Elem<T>::ld(a.q + row * a.qs + (long)h * a.D + i);
  __syncthreads();

  float acc[MAX_EPT] = {};
  float m = a.sink ? a.sink[h] : -FLT_MAX, l = a.sink ? 1.f : 0.f;
  // the kept tokens ahead of the window, then the window
  for (int part = 0; part < 2; ++part) {
    const long first = part ? lo : 0;
    const long end = part ? pos + 1 : min((long)a.keep, lo);
    for (long base = first; base < end; base += TILE) {
      const int n = (int)min((long)TILE, end - base);
      float s = -FLT_MAX;
      if (tid < n) {
        const long p = base + tid;
        const T* kp = a.k_cache +
            (((long)bt[p / PAGE] * a.G + g) * PAGE + p % PAGE) * a.D;
        float d = 0.f;
        for (int i = 0; i < a.D; ++i) d += q_lds[i] * Elem<T>::ld(kp + i);
        s = d * a.scale;
      }
      const float mn = fmaxf(m, block_reduce_max_256(s, scratch));
      const float p = tid < n ? Fn<T>::exp(s - mn) : 0.f;
      const float alpha = m == -FLT_MAX ? 0.f : Fn<T>::exp(m - mn);
      l = l * alpha + block_reduce_sum_256(p, scratch);
      m = mn;
      p_lds[tid] = p;
      __syncthreads();
      #pragma unroll
      for (int i = 0; i < MAX_EPT; ++i) {
        const int e = tid + 256 * i;
        if (e < a.E) {
          float o = acc[i] * alpha;
          for (int t = 0; t < n; ++t) {
            const long pt = base + t;
            o += p_lds[t] * Elem<T>::ld(
                a.v_cache + (((long)bt[pt / PAGE] * a.G + g) * a.E + e) *
                PAGE + pt % PAGE);
          }
          acc[i] = o;
        }
      }
      __syncthreads();
    }
  }
  #pragma unroll
  for (int i = 0; i < MAX_EPT; ++i) {
    const int e = tid + 256 * i;
    float x[2] = {acc[i] / l, 0.f};
    if (a.turn) {                       // the pair is in the next lane
      const float other = __shfl_xor(x[0], 1);
      if (e < a.E) {
        if (e & 1) { x[1] = x[0]; x[0] = other; } else { x[1] = other; }
        turn_back(a, pos, e & ~1, x);
        if (e & 1) x[0] = x[1];
      }
    }
    if (e < a.E)
      Elem<T>::st(a.out + row * a.os + (long)h * a.E + e, x[0]);
  }
}

// ============================ matrix-core prefill ==========================

constexpr int KV = 64;            // tokens per step
constexpr int VS = KV + 8;        // V^T row in LDS, padded against conflicts

// HW heads a workgroup.  Waves: row group = wave >> 1 (32 query rows each),
// and wave & 1 is the head (HW 2) or which 32 tokens of a step (HW 1).
// a.scale is in units of log2(e).
template <int DP, int EP, int HW, bool BOUNDED>
__global__ __launch_bounds__(256, DP <= 128 && EP <= 128 ? 2 : 1)
void kept_attn_prefill_kernel(Kept<bf16> a,
                              const int* __restrict__ seq_start,
                              const int* __restrict__ tiles) {
  constexpr int KS = DP + 8;                     // K row in LDS
  constexpr int KC = DP / 16, ET = EP / 32;
  constexpr int KLOADS = KV * DP / 8 / 256;      // 16-byte units a thread
  constexpr int VLOADS = KV * EP / 8 / 256;
  constexpr int NB = HW == 2 ? 2 : 1;            // 32-token blocks a wave
  constexpr int TILE_BYTES = (KV * KS + EP * VS) * 2;
  constexpr int OUT_BYTES = HW == 2 ? 0 : 2 * (EP + 2) * 32 * 4;
  constexpr int TC = EP < 128 ? EP : 128;        // columns turned at a time
  constexpr int TS = TC + 4;
  constexpr int TURN_BYTES = KV * TS * 4;
  constexpr int BYTES = TILE_BYTES > OUT_BYTES ? TILE_BYTES : OUT_BYTES;
  __shared__ __attribute__((aligned(16)))
      char smem[BYTES > TURN_BYTES ? BYTES : TURN_BYTES];
  short* k_lds = reinterpret_cast<short*>(smem);
  short* v_lds = k_lds + KV * KS;
  const int D = a.D, E = a.E, G = a.G;

  // later rows see more: they start first
  const int tile = gridDim.y - 1 - blockIdx.y;
  const int s = tiles[2 * tile];
  const int t0 = seq_start[s] + tiles[2 * tile + 1];
  const int n = min(KV, seq_start[s + 1] - t0);
  if (n <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int half = wid & 1, rg = wid >> 1;
  const int h = blockIdx.x * HW + (HW == 2 ? half : 0);
  const int g = h / (a.H / G);                   // one for both heads
  const int* bt = a.block_tables + (long)s * a.max_blocks;
  const int p0 = (int)a.positions[t0];           // rows are consecutive

  const int col = lane & 31, hf = lane >> 5;
  const int row = rg * 32 + col;                 // this lane's query row
  const int qp = p0 + row;

  short8_t qf[KC];
  {
    const bf16* qr = a.q + (long)(t0 + row) * a.qs + (long)h * D;
    #pragma unroll
    for (int c = 0; c < KC; ++c) {
      const int d = c * 16 + hf * 8;
      qf[c] = row < n && d < D
          ? *reinterpret_cast<const short8_t*>(qr + d) : short8_t{};
    }
  }
  f32x16_t acc[ET];
  #pragma unroll
  for (int e = 0; e < ET; ++e) acc[e] = f32x16_t(0.f);
  // the sink is counted once: by one half of the lanes, and of the tokens
  float m = BOUNDED ? 0.f : -FLT_MAX, l = 0.f;
  if (a.sink) {
    const float s = a.sink[h] * LOG2E;
    if (!BOUNDED) m = s;
    if (hf == 0 && (HW == 2 || half == 0)) l = exp2_fast(s - m);
  }

  const int last = p0 + n - 1;
  // rows of this wave
  const int w_first = p0 + rg * 32, w_last = min(w_first + 31, last);
  // the steps: kept tokens, then from the first row's window on
  const int from = max(0, p0 - a.window + 1) / KV * KV;
  const int kept = min(a.keep, last + 1);
  auto next = [&](int kv) {
    kv += KV;
    return kv >= kept && kv < from ? from : kv;
  };

  uint4 kr[KLOADS], vr[VLOADS];
  // a step's four page ids are read one step ahead of its K and V loads
  int4 ids;
  auto pages = [&](int kv0) {
    ids.x = bt[min(kv0, last) / PAGE];
    ids.y = bt[min(kv0 + PAGE, last) / PAGE];
    ids.z = bt[min(kv0 + 2 * PAGE, last) / PAGE];
    ids.w = bt[min(kv0 + 3 * PAGE, last) / PAGE];
  };
  auto fetch = [&](int kv0) {
    const int i0 = ids.x, i1 = ids.y, i2 = ids.z, i3 = ids.w;
    const int after = next(kv0);
    if (after <= last) pages(after);
    auto page = [=](int j) -> long {
      const int even = (j & 1) ? i1 : i0, odd = (j & 1) ? i3 : i2;
      return (j & 2) ? odd : even;
    };
    #pragma unroll
    for (int i = 0; i < KLOADS; ++i) {
      const int u = tid + 256 * i;
      const int r = u / (DP / 8), k = (u % (DP / 8)) * 8;
      kr[i] = uint4{0, 0, 0, 0};
      if (k < D && kv0 + r <= last)
        kr[i] = *reinterpret_cast<const uint4*>(
            a.k_cache + ((page(r / PAGE) * G + g) * PAGE + r % PAGE) * D + k);
    }
    #pragma unroll
    for (int i = 0; i < VLOADS; ++i) {
      const int u = tid + 256 * i;
      const int pg = u / (EP * 2), e = (u / 2) % EP, part = u & 1;
      vr[i] = uint4{0, 0, 0, 0};
      if (e < E && kv0 + pg * PAGE <= last)
        vr[i] = *reinterpret_cast<const uint4*>(
            a.v_cache + ((page(pg) * G + g) * E + e) * PAGE + part * 8);
    }
  };
  auto stage = [&]() {
    #pragma unroll
    for (int i = 0; i < KLOADS; ++i) {
      const int u = tid + 256 * i;
      *reinterpret_cast<uint4*>(
          k_lds + (u / (DP / 8)) * KS + (u % (DP / 8)) * 8) = kr[i];
    }
    #pragma unroll
    for (int i = 0; i < VLOADS; ++i) {
      const int u = tid + 256 * i;
      const int pg = u / (EP * 2), e = (u / 2) % EP, part = u & 1;
      *reinterpret_cast<uint4*>(v_lds + e * VS + pg * PAGE + part * 8) =
          vr[i];
    }
  };

  // matrix row i of a 32-token block takes this token's key
  const int krow = (col & 16) + ((col >> 2) & 1) * 8 + ((col >> 3) & 1) * 4 +
                   (col & 3);
  // NB blocks from token kb on; FULL: every row sees all of them
  auto step = [&](int kb, auto full) {
    constexpr bool FULL = decltype(full)::value;
    const int b0 = HW == 2 ? 0 : half;           // first block in LDS
    f32x16_t sc[NB];
    auto scores = [&](int i) {
      sc[i] = f32x16_t(0.f);
      #pragma unroll
      for (int c = 0; c < KC; ++c)
        sc[i] = mfma32(*reinterpret_cast<const short8_t*>(
                           k_lds + ((b0 + i) * 32 + krow) * KS + c * 16 +
                           hf * 8),
                       qf[c], sc[i]);
      // token of sc[i][r]: kb + i*32 + (r>>3)*16 + hf*8 + (r&7)
      #pragma unroll
      for (int r = 0; r < 16; ++r) {
        float x = sc[i][r] * a.scale;
        if constexpr (!FULL) {
          const int at = kb + i * 32 + (r >> 3) * 16 + hf * 8 + (r & 7);
          if (at > qp || (at <= qp - a.window && at >= a.keep)) x = -FLT_MAX;
        }
        sc[i][r] = x;
      }
    };
    auto values = [&](int i, float base) {
      short8_t ph[2], pl[2];
      #pragma unroll
      for (int c = 0; c < 2; ++c) {
        float p[8];
        #pragma unroll
        for (int j = 0; j < 8; ++j) {
          p[j] = exp2_fast(BOUNDED ? sc[i][c * 8 + j]
                                   : sc[i][c * 8 + j] - base);
          l += p[j];
        }
        split_bf16x8(p, &ph[c], &pl[c]);
      }
      #pragma unroll
      for (int e = 0; e < ET; ++e)
        #pragma unroll
        for (int c = 0; c < 2; ++c) {
          const short8_t vf = *reinterpret_cast<const short8_t*>(
              v_lds + (e * 32 + col) * VS + (b0 + i) * 32 + c * 16 + hf * 8);
          acc[e] = mfma32(vf, ph[c], acc[e]);
          acc[e] = mfma32(vf, pl[c], acc[e]);
        }
    };
    if constexpr (BOUNDED) {
      #pragma unroll
      for (int i = 0; i < NB; ++i) {
        scores(i);
        values(i, 0.f);
      }
    } else {
      float mx = m;
      #pragma unroll
      for (int i = 0; i < NB; ++i) {
        scores(i);
        #pragma unroll
        for (int r = 0; r < 16; ++r) mx = fmaxf(mx, sc[i][r]);
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
      #pragma unroll
      for (int i = 0; i < NB; ++i) values(i, base);
    }
  };
  int kv0 = kept > 0 ? 0 : from;
  pages(kv0);
  fetch(kv0);
  while (kv0 <= last) {
    const int after = next(kv0);
    stage();
    __syncthreads();
    if (after <= last) fetch(after);
    const int kb = kv0 + (HW == 2 ? 0 : half * 32);    // first token
    const int ke = kb + NB * 32;                       // past the last one
    if (w_first <= last && kb <= w_last &&
        (ke > w_first - a.window + 1 || kb < a.keep)) {
      if (ke <= w_first + 1 && (kb > w_last - a.window || ke <= a.keep))
        step(kb, std::true_type{});
      else
        step(kb, std::false_type{});
    }
    __syncthreads();
    kv0 = after;
  }
  l += __shfl_xor(l, 32);

  if constexpr (HW == 1) {          // the two halves of the tokens meet
    float* o_lds = reinterpret_cast<float*>(smem);   // [2][EP + 2][32]
    float* ml = o_lds + 2 * EP * 32;
    if (half == 1) {
      #pragma unroll
      for (int e = 0; e < ET; ++e)
        #pragma unroll
        for (int r = 0; r < 16; ++r)
          o_lds[((rg * ET + e) * 16 + r) * 64 + lane] = acc[e][r];
      if (hf == 0) {
        ml[(rg * 2) * 32 + col] = m;
        ml[(rg * 2 + 1) * 32 + col] = l;
      }
    }
    __syncthreads();
    if (half == 0) {
      const float m1 = ml[(rg * 2) * 32 + col];
      const float l1 = ml[(rg * 2 + 1) * 32 + col];
      const float top = fmaxf(m, m1);
      const float w0 = m == -FLT_MAX ? 0.f : exp2_fast(m - top);
      const float w1 = m1 == -FLT_MAX ? 0.f : exp2_fast(m1 - top);
      l = l * w0 + l1 * w1;
      #pragma unroll
      for (int e = 0; e < ET; ++e)
        #pragma unroll
        for (int r = 0; r < 16; ++r)
          acc[e][r] = acc[e][r] * w0 +
                      o_lds[((rg * ET + e) * 16 + r) * 64 + lane] * w1;
    }
  }
  const bool writes = row < n && (HW == 2 || half == 0);
  const float inv = 1.f / l;
  bf16* orow = a.out + (long)(t0 + row) * a.os + (long)h * E;
  float* cs_lds = reinterpret_cast<float*>(smem);    // [KV][TS] (cos, sin)
  #pragma unroll
  for (int e0 = 0; e0 < ET; e0 += TC / 32) {
    if (a.turn) {                     // the rows' angles, for all heads here
      __syncthreads();
      for (int u = tid; u < KV * (TC / 2); u += 256) {
        const int r = u / (TC / 2), i = u % (TC / 2);
        if (e0 * 32 + 2 * i < E)
          angle<bf16>(-(long)(p0 + r), a.turn[e0 * 16 + i],
                      &cs_lds[r * TS + 2 * i], &cs_lds[r * TS + 2 * i + 1]);
      }
      __syncthreads();
    }
    if (!writes) continue;
    #pragma unroll
    for (int e = e0; e < e0 + TC / 32; ++e)
      #pragma unroll
      for (int r = 0; r < 16; r += 4) {
        const int c = e * 32 + 8 * (r >> 2) + 4 * hf;
        if (c >= E) continue;
        float x[4];
        #pragma unroll
        for (int i = 0; i < 4; ++i) x[i] = acc[e][r + i] * inv;
        if (a.turn) {
          float cs[4];
          load_vec<float, 4>(cs_lds + row * TS + c - e0 * 32, cs);
          turn_pairs<4>(x, cs);
        }
        *reinterpret_cast<uint2*>(orow + c) =
            uint2{cvt_pk_bf16(x[0], x[1]), cvt_pk_bf16(x[2], x[3])};
      }
  }
}

// ============================ matrix-core decode ===========================
constexpr int NC = 16;            // query heads per workgroup, at most
constexpr int PART = 4;           // floats past the values of a part: m, l

// a.scale is in units of log2(e)
template <int DP, int EP, bool BOUNDED>
__global__ __launch_bounds__(256, DP <= 128 && EP <= 128 ? 2 : 1)
void kept_attn_decode_kernel(Kept<bf16> a, float* __restrict__ partial) {
  constexpr int KC = (DP + 31) / 32, ET = EP / 16;
  extern __shared__ float m_lds[];  // [4 waves][NC], as many sums after them
  float* l_lds = m_lds + 4 * NC;
  float* comb = l_lds + 4 * NC;     // [4 waves][cols][E]
  const int D = a.D, E = a.E, G = a.G, H = a.H;
  const long row = blockIdx.x;
  const int group = H / G, hb = (group + NC - 1) / NC;
  const int g = blockIdx.y / hb;
  const int h0 = g * group + (blockIdx.y % hb) * NC;
  const int cols = min(NC, group - (blockIdx.y % hb) * NC);
  const int split = gridDim.z, z = blockIdx.z;
  const int* bt = a.block_tables + row * a.max_blocks;
  const int pos = (int)a.positions[row];
  const int lo = max(0, pos - a.window + 1);
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int col = lane & 15, gr = lane >> 4;

  short8_t qf[KC];
  #pragma unroll
  for (int c = 0; c < KC; ++c) {
    const int d = c * 32 + gr * 8;
    qf[c] = col < cols && d < D
        ? *reinterpret_cast<const short8_t*>(
              a.q + row * a.qs + (long)(h0 + col) * D + d)
        : short8_t{};
  }
  f32x4_t acc[ET];
  #pragma unroll
  for (int e = 0; e < ET; ++e) acc[e] = f32x4_t(0.f);
  // the sink is counted once: by one part, wave and quarter of the lanes
  float m = BOUNDED ? 0.f : -FLT_MAX, l = 0.f;
  if (a.sink && z == 0 && wid == 0) {
    const float s = a.sink[h0 + min(col, cols - 1)] * LOG2E;
    if (!BOUNDED) m = s;
    if (gr == 0) l = exp2_fast(s - m);
  }

  // blocks of 32 tokens: kept ones ahead of the window's first, then those of
  // the window; this wave takes every (4 split)-th
  const int wb = lo / 32;
  const int kb = min((min(a.keep, pos + 1) + 31) / 32, wb);
  const int blocks = kb + pos / 32 - wb + 1;
  auto first_of = [&](int i) { return (i < kb ? i : wb + i - kb) * 32; };
  // matrix row i of half-block t takes token 8*(i>>2) + 4*t + (i&3)
  const int tok0 = 8 * (col >> 2) + (col & 3);
  int i = z * 4 + wid;
  long b0 = 0, b1 = 0;               // page ids, read one block ahead
  auto pages = [&](int i) {
    const int p0 = first_of(i);
    b0 = bt[p0 / PAGE];
    b1 = bt[min(p0 + PAGE, pos) / PAGE];
  };
  if (i < blocks) pages(i);
  for (; i < blocks; i += split * 4) {
    const int p0 = first_of(i);
    short8_t kf[2][KC];
    #pragma unroll
    for (int t = 0; t < 2; ++t) {
      const int tok = tok0 + 4 * t;
      const bf16* kp = a.k_cache +
          (((tok < PAGE ? b0 : b1) * G + g) * PAGE + tok % PAGE) * D;
      #pragma unroll
      for (int c = 0; c < KC; ++c) {
        const int d = c * 32 + gr * 8;
        kf[t][c] = d < D ? *reinterpret_cast<const short8_t*>(kp + d)
                         : short8_t{};
      }
    }
    short8_t vf[ET];
    const bf16* vp = a.v_cache +
        ((gr < 2 ? b0 : b1) * G + g) * (long)E * PAGE + (gr & 1) * 8;
    #pragma unroll
    for (int e = 0; e < ET; ++e)
      vf[e] = e * 16 + col < E
          ? *reinterpret_cast<const short8_t*>(vp + (e * 16 + col) * PAGE)
          : short8_t{};
    if (i + split * 4 < blocks) pages(i + split * 4);
    const int tp = p0 + gr * 8;       // this lane's 8 consecutive tokens
    f32x4_t sc[2];
    #pragma unroll
    for (int t = 0; t < 2; ++t) {
      sc[t] = f32x4_t(0.f);
      #pragma unroll
      for (int c = 0; c < KC; ++c) sc[t] = mfma16(kf[t][c], qf[c], sc[t]);
    }
    float p[8], mx = m;
    #pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int at = tp + j;
      p[j] = at <= pos && (at >= lo || at < a.keep)
          ? sc[j >> 2][j & 3] * a.scale : -FLT_MAX;
      if constexpr (!BOUNDED) mx = fmaxf(mx, p[j]);
    }
    if constexpr (!BOUNDED) {
      mx = fmaxf(mx, __shfl_xor(mx, 16));
      mx = fmaxf(mx, __shfl_xor(mx, 32));
      if (!__all(mx == m)) {
        const float alpha = m == -FLT_MAX ? 0.f : exp2_fast(m - mx);
        #pragma unroll
        for (int e = 0; e < ET; ++e)
          #pragma unroll
          for (int r = 0; r < 4; ++r) acc[e][r] *= alpha;
        l *= alpha;
        m = mx;
      }
    }
    const float base = BOUNDED || m == -FLT_MAX ? 0.f : m;
    #pragma unroll
    for (int j = 0; j < 8; ++j) {
      p[j] = exp2_fast(BOUNDED ? p[j] : p[j] - base);
      l += p[j];
    }
    short8_t ph, pl;
    split_bf16x8(p, &ph, &pl);
    #pragma unroll
    for (int e = 0; e < ET; ++e) {
      acc[e] = mfma16(vf[e], ph, acc[e]);
      acc[e] = mfma16(vf[e], pl, acc[e]);
    }
  }
  l += __shfl_xor(l, 16);
  l += __shfl_xor(l, 32);
  if (gr == 0) {
    m_lds[wid * NC + col] = m;
    l_lds[wid * NC + col] = l;
  }
  if (col < cols) {
    float* c = comb + (wid * cols + col) * E;
    #pragma unroll
    for (int e = 0; e < ET; ++e)
      if (e * 16 + gr * 4 < E)        // E is a multiple of 8
        *reinterpret_cast<f32x4_t*>(c + e * 16 + gr * 4) = acc[e];
  }
  __syncthreads();
  const int n = cols * E;
  for (int u = tid * 4; u < n; u += 1024) {
    const int hc = u / E, c = u % E;
    float top = -FLT_MAX, sum = 0.f;
    #pragma unroll
    for (int w = 0; w < 4; ++w) top = fmaxf(top, m_lds[w * NC + hc]);
    f32x4_t o = f32x4_t(0.f);
    #pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float mw = m_lds[w * NC + hc];
      const float f = mw == -FLT_MAX ? 0.f : exp2_fast(mw - top);
      sum += f * l_lds[w * NC + hc];
      o += *reinterpret_cast<const f32x4_t*>(comb + w * n + u) * f;
    }
    const int h = h0 + hc;
    if (split == 1) {
      float x[4];
      #pragma unroll
      for (int j = 0; j < 4; ++j) x[j] = o[j] / sum;
      if (a.turn) {
        turn_back(a, pos, c, x);
        turn_back(a, pos, c + 2, x + 2);
      }
      *reinterpret_cast<uint2*>(a.out + row * a.os + (long)h * E + c) =
          uint2{cvt_pk_bf16(x[0], x[1]), cvt_pk_bf16(x[2], x[3])};
    } else {
      float* dst = partial + ((row * H + h) * split + z) * (long)(E + PART);
      *reinterpret_cast<f32x4_t*>(dst + c) = o;
      if (c == 0) {
        dst[E] = top;
        dst[E + 1] = sum;
      }
    }
  }
}

// the parts of a row combined, 4 of its H * E columns a thread
__global__ __launch_bounds__(256) void kept_attn_merge_kernel(
    Kept<bf16> a, const float* __restrict__ partial, int split) {
  const int u = (blockIdx.y * 256 + threadIdx.x) * 4;
  if (u >= a.H * a.E) return;
  const long row = blockIdx.x;
  const int h = u / a.E, c = u % a.E, width = a.E + PART;
  const float* src = partial + (row * a.H + h) * split * (long)width;
  float top = -FLT_MAX, sum = 0.f;
  #pragma unroll 4
  for (int z = 0; z < split; ++z) top = fmaxf(top, src[(long)z * width + a.E]);
  f32x4_t o = f32x4_t(0.f);
  #pragma unroll 4
  for (int z = 0; z < split; ++z) {
    const float* p = src + (long)z * width;
    const float f = p[a.E] == -FLT_MAX ? 0.f : exp2_fast(p[a.E] - top);
    sum += f * p[a.E + 1];
    o += *reinterpret_cast<const f32x4_t*>(p + c) * f;
  }
  float x[4];
  #pragma unroll
  for (int j = 0; j < 4; ++j) x[j] = o[j] / sum;
  if (a.turn) {
    turn_back(a, a.positions[row], c, x);
    turn_back(a, a.positions[row], c + 2, x + 2);
  }
  *reinterpret_cast<uint2*>(a.out + row * a.os + u) =
      uint2{cvt_pk_bf16(x[0], x[1]), cvt_pk_bf16(x[2], x[3])};
}

}  // namespace

template <typename T>
void launch_kept_attn_general(T* out, const T* q, const T* k_cache,
                              const T* v_cache, const int* block_tables,
                              const long* positions, const int* row_seq,
                              const double* turn, const float* sink,
                              long rows, int max_blocks, int H, int G, int D,
                              int E, int window, int keep, float scale,
                              long qs, long os, hipStream_t stream) {
  if (rows == 0) return;
  const Kept<T> a{out, q, k_cache, v_cache, block_tables, positions, turn,
                  sink, max_blocks, H, G, D, E, window, keep, scale, qs, os};
  kept_attn_general_kernel<T>
      <<<dim3((unsigned)rows, (unsigned)H), 256, (D + TILE) * sizeof(float),
         stream>>>(a, row_seq);
}
template void launch_kept_attn_general<bf16>(
    bf16*, const bf16*, const bf16*, const bf16*, const int*, const long*,
    const int*, const double*, const float*, long, int, int, int, int, int,
    int, int, float, long, long, hipStream_t);
template void launch_kept_attn_general<float>(
    float*, const float*, const float*, const float*, const int*,
    const long*, const int*, const double*, const float*, long, int, int,
    int, int, int, int, int, float, long, long, hipStream_t);

// padded sizes of the matrix-core kernels
#define KEPT_SIZES(CASE)                                                    \
  CASE(64, 64) CASE(64, 128) CASE(128, 128) CASE(64, 256) CASE(128, 256)    \
  CASE(256, 256)

void launch_kept_attn_prefill(bf16* out, const bf16* q, const bf16* k_cache,
                              const bf16* v_cache, const int* block_tables,
                              const long* positions, const int* seq_start,
                              const int* tiles, const double* turn,
                              const float* sink, int num_tiles,
                              int max_blocks, int H, int G, int D, int E,
                              int window, int keep, float scale, bool bounded,
                              long qs, long os, hipStream_t stream) {
  if (num_tiles == 0) return;
  const Kept<bf16> a{out, q, k_cache, v_cache, block_tables, positions, turn,
                     sink, max_blocks, H, G, D, E, window, keep,
                     scale * LOG2E, qs, os};
  // two heads share a tile's keys where enough workgroups remain
  const int hw = H / G % 2 == 0 && (long)H / 2 * num_tiles >= 512 ? 2 : 1;
  const dim3 grid((unsigned)(H / hw), (unsigned)num_tiles);
  #define RUN(DP, EP, HW, BOUNDED)                                          \
    kept_attn_prefill_kernel<DP, EP, HW, BOUNDED>                           \
        <<<grid, 256, 0, stream>>>(a, seq_start, tiles)
  #define CASE(DP, EP)                                                      \
    if (D <= DP && E <= EP) {                                               \
      if (hw == 2) {                                                        \
        if (bounded) RUN(DP, EP, 2, true); else RUN(DP, EP, 2, false);      \
      } else {                                                              \
        if (bounded) RUN(DP, EP, 1, true); else RUN(DP, EP, 1, false);      \
      }                                                                     \
      return;                                                               \
    }
  KEPT_SIZES(CASE)
  #undef CASE
  #undef RUN
  throw std::runtime_error("kept_attn_prefill: head sizes");
}

void launch_kept_attn_decode(bf16* out, const bf16* q, const bf16* k_cache,
                             const bf16* v_cache, const int* block_tables,
                             const long* positions, const double* turn,
                             const float* sink, float* partial, long rows,
                             int max_blocks, int H, int G, int D, int E,
                             int window, int keep, float scale, bool bounded,
                             long qs, long os, int split,
                             hipStream_t stream) {
  if (rows == 0) return;
  const Kept<bf16> a{out, q, k_cache, v_cache, block_tables, positions, turn,
                     sink, max_blocks, H, G, D, E, window, keep,
                     scale * LOG2E, qs, os};
  const int group = H / G, hb = (group + NC - 1) / NC;
  const int cols = group < NC ? group : NC;
  const int lds = (4 * cols * E + 8 * NC) * (int)sizeof(float);
  const dim3 grid((unsigned)rows, (unsigned)(G * hb), (unsigned)split);
  auto run = [&](auto kernel) {
    if (lds > 65536)
      HIP_CHECK(hipFuncSetAttribute(
          reinterpret_cast<const void*>(kernel),
          hipFuncAttributeMaxDynamicSharedMemorySize, lds));
    kernel<<<grid, 256, lds, stream>>>(a, partial);
    if (split > 1)
      kept_attn_merge_kernel<<<
          dim3((unsigned)rows, (unsigned)((H * E + 1023) / 1024)), 256, 0,
          stream>>>(a, partial, split);
  };
  #define CASE(DP, EP)                                                      \
    if (D <= DP && E <= EP)                                                 \
      return bounded ? run(&kept_attn_decode_kernel<DP, EP, true>)          \
                     : run(&kept_attn_decode_kernel<DP, EP, false>);
  KEPT_SIZES(CASE)
  #undef CASE
  throw std::runtime_error("kept_attn_decode: head sizes");
}
