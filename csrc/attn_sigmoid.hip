// Chunked sigmoid attention over the paged cache (gfx950).
//
// Row t of position p sees the positions p - p % chunk ... p of its sequence.
// A key weighs sigmoid(cap * tanh(q.k * scale / cap) + bias[h]); weights are
// not normalized over keys, so there is no running maximum, and partial sums
// over any split of the keys just add up.
//
//   q       [T, H * D]  (token stride qs)       out [T, H * E]
//   k_cache [NB, G, 16, D]     v_cache [NB, G, E, 16]  (V^T per page)
//
// Three kernels:
//   general  any head sizes, bf16 or float, prefill and decode rows alike, one
//            workgroup per (row, head);
//   prefill  bf16 matrix cores, 64 query rows of one or two heads a workgroup;
//   decode   bf16 matrix cores, one row and up to 16 heads of a kv head a
//            workgroup, optionally split over the chunk with a merge pass.
// The matrix-core kernels want D and E to be multiples of 8, at most 256;
// smaller sizes are padded with zeros in registers and LDS.
//
// Operand layouts (v_mfma_f32_32x32x16 / 16x16x32, bf16):  scores are formed
// transposed, S^T = K Q^T, with the K row that feeds matrix row i permuted so
// that the scores a lane holds are 8 consecutive tokens of one query column,
// which is the operand P^T of O^T = V^T P^T: weights never leave their
// registers, and V^T comes straight from the transposed pages.  The weights
// enter as a bf16 high and low part.
#include <type_traits>

#include "common.h"

#define PAGE 16

namespace {

constexpr int TILE = 256;      // tokens per step of the general kernel
constexpr int MAX_EPT = 4;     // values per thread: E <= 1024

template <typename T>
__global__ __launch_bounds__(256) void sigmoid_attn_general_kernel(
    T* __restrict__ out, const T* __restrict__ q,
    const T* __restrict__ k_cache, const T* __restrict__ v_cache,
    const int* __restrict__ block_tables, const long* __restrict__ positions,
    const int* __restrict__ row_seq, const float* __restrict__ bias,
    int max_blocks, int H, int G, int D, int E, int chunk, float scale,
    float cap, long qs) {
  extern __shared__ float smem[];
  float* q_lds = smem;                 // [D]
  float* p_lds = smem + D;             // [TILE]
  const long row = blockIdx.x;
  const int h = blockIdx.y, g = h / (H / G), tid = threadIdx.x;
  const int* bt = block_tables +
                  (long)(row_seq ? row_seq[row] : (int)row) * max_blocks;
  const long pos = positions[row];
  for (int i = tid; i < D; i += 256)
    q_lds[i] = Elem<T>::ld(q + row * qs + (long)h * D + i);
  __syncthreads();

  float acc[MAX_EPT] = {};
  for (long base = pos - pos % chunk; base <= pos; base += TILE) {
    const int n = (int)min((long)TILE, pos - base + 1);
    if (tid < n) {
      const long p = base + tid;
      const T* kp = k_cache +
          (((long)bt[p / PAGE] * G + g) * PAGE + p % PAGE) * D;
      float d = 0.f;
      for (int i = 0; i < D; ++i) d += q_lds[i] * Elem<T>::ld(kp + i);
      const float z = cap * Fn<T>::tanh(d * scale / cap) + bias[h];
      p_lds[tid] = 1.f / (1.f + Fn<T>::exp(-z));
    }
    __syncthreads();
    #pragma unroll
    for (int i = 0; i < MAX_EPT; ++i) {
      const int e = tid + 256 * i;
      if (e < E)
        for (int t = 0; t < n; ++t) {
          const long p = base + t;
          acc[i] += p_lds[t] * Elem<T>::ld(
              v_cache + (((long)bt[p / PAGE] * G + g) * E + e) * PAGE +
              p % PAGE);
        }
    }
    __syncthreads();
  }
  #pragma unroll
  for (int i = 0; i < MAX_EPT; ++i)
    if (tid + 256 * i < E)
      Elem<T>::st(out + (row * H + h) * E + tid + 256 * i, acc[i]);
}

// weight of a raw score s: with u = s * scale / cap,
//   -z / ln 2 = a + b / (1 + e^(2u)),  a = -(cap + bias) / ln 2,
//   b = 2 cap / ln 2,   weight = 1 / (1 + 2^(-z / ln 2))
struct Weigh {
  float k, a, b;

  DEV Weigh(float scale, float cap, float bias) {
    constexpr float LOG2E = 1.4426950408889634f;
    k = 2.f * LOG2E * scale / cap;
    a = -(cap + bias) * LOG2E;
    b = 2.f * cap * LOG2E;
  }
  DEV float operator()(float s) const {
    const float t =
        __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(k * s));
    return __builtin_amdgcn_rcpf(
        1.f + __builtin_amdgcn_exp2f(__builtin_fmaf(b, t, a)));
  }
};

// ============================ matrix-core prefill ==========================

constexpr int KV = 64;            // tokens per step
constexpr int VS = KV + 8;        // V^T row in LDS, padded against conflicts

// HW heads a workgroup.  Waves: row group = wave >> 1 (32 query rows each),
// and wave & 1 is the head (HW 2) or which 32 tokens of a step (HW 1).
template <int DP, int EP, int HW>
__global__ __launch_bounds__(256, DP <= 128 && EP <= 128 ? 2 : 1)
void sigmoid_attn_prefill_kernel(
    bf16* __restrict__ out, const bf16* __restrict__ q,
    const bf16* __restrict__ k_cache, const bf16* __restrict__ v_cache,
    const int* __restrict__ block_tables, const long* __restrict__ positions,
    const int* __restrict__ seq_start, const int* __restrict__ tiles,
    const float* __restrict__ bias, int max_blocks, int H, int G, int D,
    int E, int chunk, float scale, float cap, long qs) {
  constexpr int KS = DP + 8;                     // K row in LDS
  constexpr int KC = DP / 16, ET = EP / 32;
  constexpr int KLOADS = KV * DP / 8 / 256;      // 16-byte units a thread
  constexpr int VLOADS = KV * EP / 8 / 256;
  constexpr int NB = HW == 2 ? 2 : 1;            // 32-token blocks a wave
  constexpr int TILE_BYTES = (KV * KS + EP * VS) * 2;
  constexpr int OUT_BYTES = HW == 2 ? 0 : 2 * EP * 32 * 4;
  __shared__ __attribute__((aligned(16)))
      char smem[TILE_BYTES > OUT_BYTES ? TILE_BYTES : OUT_BYTES];
  short* k_lds = reinterpret_cast<short*>(smem);
  short* v_lds = k_lds + KV * KS;

  // later rows see more: they start first
  const int tile = gridDim.y - 1 - blockIdx.y;
  const int s = tiles[2 * tile];
  const int first = tiles[2 * tile + 1];
  const int t0 = seq_start[s] + first;
  const int n = min(KV, seq_start[s + 1] - t0);
  if (n <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int half = wid & 1, rg = wid >> 1;
  const int h = blockIdx.x * HW + (HW == 2 ? half : 0);
  const int g = h / (H / G);                     // one for both heads
  const int* bt = block_tables + (long)s * max_blocks;
  const int p0 = (int)positions[t0];             // rows are consecutive

  const int col = lane & 31, hf = lane >> 5;
  const int row = rg * 32 + col;                 // this lane's query row
  const int qp = p0 + row;
  const int q_lo = qp - qp % chunk;              // first visible position

  short8_t qf[KC];
  {
    const bf16* qr = q + (long)(t0 + row) * qs + (long)h * D;
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
  const Weigh weigh(scale, cap, bias[h]);

  const int last = p0 + n - 1;
  // rows of this wave: first and last position and what they see
  const int w_first = p0 + rg * 32, w_last = min(w_first + 31, last);
  const int w_lo = w_first - w_first % chunk, w_hi = w_last - w_last % chunk;

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
    const int a = ids.x, b = ids.y, c = ids.z, d = ids.w;
    if (kv0 + KV <= last) pages(kv0 + KV);
    auto page = [=](int j) -> long {
      const int lo = (j & 1) ? b : a, hi = (j & 1) ? d : c;
      return (j & 2) ? hi : lo;
    };
    #pragma unroll
    for (int i = 0; i < KLOADS; ++i) {
      const int u = tid + 256 * i;
      const int r = u / (DP / 8), k = (u % (DP / 8)) * 8;
      kr[i] = uint4{0, 0, 0, 0};
      if (k < D && kv0 + r <= last)
        kr[i] = *reinterpret_cast<const uint4*>(
            k_cache + ((page(r / PAGE) * G + g) * PAGE + r % PAGE) * D + k);
    }
    #pragma unroll
    for (int i = 0; i < VLOADS; ++i) {
      const int u = tid + 256 * i;
      const int pg = u / (EP * 2), e = (u / 2) % EP, part = u & 1;
      vr[i] = uint4{0, 0, 0, 0};
      if (e < E && kv0 + pg * PAGE <= last)
        vr[i] = *reinterpret_cast<const uint4*>(
            v_cache + ((page(pg) * G + g) * E + e) * PAGE + part * 8);
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
    #pragma unroll
    for (int i = 0; i < NB; ++i) {
      sc[i] = f32x16_t(0.f);
      #pragma unroll
      for (int c = 0; c < KC; ++c)
        sc[i] = mfma32(*reinterpret_cast<const short8_t*>(
                           k_lds + ((b0 + i) * 32 + krow) * KS + c * 16 +
                           hf * 8),
                       qf[c], sc[i]);
    }
    #pragma unroll
    for (int i = 0; i < NB; ++i) {
      // token of sc[i][r]: kb + i*32 + (r>>3)*16 + hf*8 + (r&7)
      short8_t ph[2], pl[2];
      #pragma unroll
      for (int c = 0; c < 2; ++c) {
        float p[8];
        #pragma unroll
        for (int j = 0; j < 8; ++j) {
          p[j] = weigh(sc[i][c * 8 + j]);
          if constexpr (!FULL) {
            const int at = kb + i * 32 + c * 16 + hf * 8 + j;
            if (at > qp || at < q_lo) p[j] = 0.f;
          }
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
    }
  };
  const int kv_first = (p0 - p0 % chunk) / KV * KV;
  pages(kv_first);
  fetch(kv_first);
  for (int kv0 = kv_first; kv0 <= last; kv0 += KV) {
    stage();
    __syncthreads();
    if (kv0 + KV <= last) fetch(kv0 + KV);
    const int kb = kv0 + (HW == 2 ? 0 : half * 32);    // first token
    if (w_first <= last && kb <= w_last && kb + NB * 32 > w_lo) {
      if (kb + NB * 32 <= w_first + 1 && kb >= w_hi)
        step(kb, std::true_type{});
      else
        step(kb, std::false_type{});
    }
    __syncthreads();
  }

  if constexpr (HW == 1) {          // the two halves of the tokens meet
    float* o_lds = reinterpret_cast<float*>(smem);
    if (half == 1) {
      #pragma unroll
      for (int e = 0; e < ET; ++e)
        #pragma unroll
        for (int r = 0; r < 16; ++r)
          o_lds[((rg * ET + e) * 16 + r) * 64 + lane] = acc[e][r];
    }
    __syncthreads();
    if (half == 1) return;
    #pragma unroll
    for (int e = 0; e < ET; ++e)
      #pragma unroll
      for (int r = 0; r < 16; ++r)
        acc[e][r] += o_lds[((rg * ET + e) * 16 + r) * 64 + lane];
  }
  if (row >= n) return;
  bf16* orow = out + ((long)(t0 + row) * H + h) * E;
  #pragma unroll
  for (int e = 0; e < ET; ++e)
    #pragma unroll
    for (int r = 0; r < 16; r += 4) {
      const int c = e * 32 + 8 * (r >> 2) + 4 * hf;
      if (c < E)
        *reinterpret_cast<uint2*>(orow + c) = uint2{
            cvt_pk_bf16(acc[e][r], acc[e][r + 1]),
            cvt_pk_bf16(acc[e][r + 2], acc[e][r + 3])};
    }
}

// ============================ matrix-core decode ===========================
constexpr int NC = 16;            // query heads per workgroup, at most

template <int DP, int EP>
__global__ __launch_bounds__(256, DP <= 128 && EP <= 128 ? 2 : 1)
void sigmoid_attn_decode_kernel(
    bf16* __restrict__ out, const bf16* __restrict__ q,
    const bf16* __restrict__ k_cache, const bf16* __restrict__ v_cache,
    const int* __restrict__ block_tables, const long* __restrict__ positions,
    const float* __restrict__ bias, float* __restrict__ partial,
    int max_blocks, int H, int G, int D, int E, int chunk, float scale,
    float cap, long qs) {
  constexpr int KC = (DP + 31) / 32, ET = EP / 16;
  extern __shared__ float comb[];   // [4 waves][cols][E]
  const long row = blockIdx.x;
  const int group = H / G, hb = (group + NC - 1) / NC;
  const int g = blockIdx.y / hb;
  const int h0 = g * group + (blockIdx.y % hb) * NC;
  const int cols = min(NC, group - (blockIdx.y % hb) * NC);
  const int split = gridDim.z, z = blockIdx.z;
  const int* bt = block_tables + row * max_blocks;
  const int pos = (int)positions[row];
  const int lo = pos - pos % chunk;
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int col = lane & 15, gr = lane >> 4;

  short8_t qf[KC];
  #pragma unroll
  for (int c = 0; c < KC; ++c) {
    const int d = c * 32 + gr * 8;
    qf[c] = col < cols && d < D
        ? *reinterpret_cast<const short8_t*>(
              q + row * qs + (long)(h0 + col) * D + d)
        : short8_t{};
  }
  f32x4_t acc[ET];
  #pragma unroll
  for (int e = 0; e < ET; ++e) acc[e] = f32x4_t(0.f);
  const Weigh weigh(scale, cap, bias[h0 + min(col, cols - 1)]);

  // matrix row i of half-block t takes token 8*(i>>2) + 4*t + (i&3)
  const int tok0 = 8 * (col >> 2) + (col & 3);
  for (int p0 = (lo / 32 + z * 4 + wid) * 32; p0 <= pos;
       p0 += split * 4 * 32) {
    const long b0 = bt[p0 / PAGE];
    const long b1 = p0 + PAGE <= pos ? bt[p0 / PAGE + 1] : b0;
    short8_t kf[2][KC];
    #pragma unroll
    for (int t = 0; t < 2; ++t) {
      const int tok = tok0 + 4 * t;
      const bf16* kp = k_cache +
          (((tok < PAGE ? b0 : b1) * G + g) * PAGE + tok % PAGE) * D;
      #pragma unroll
      for (int c = 0; c < KC; ++c) {
        const int d = c * 32 + gr * 8;
        kf[t][c] = d < D ? *reinterpret_cast<const short8_t*>(kp + d)
                         : short8_t{};
      }
    }
    short8_t vf[ET];
    const bf16* vp = v_cache + ((gr < 2 ? b0 : b1) * G + g) * (long)E * PAGE
                     + (gr & 1) * 8;
    #pragma unroll
    for (int e = 0; e < ET; ++e)
      vf[e] = e * 16 + col < E
          ? *reinterpret_cast<const short8_t*>(vp + (e * 16 + col) * PAGE)
          : short8_t{};
    const int tp = p0 + gr * 8;       // this lane's 8 consecutive tokens
    f32x4_t sc[2];
    #pragma unroll
    for (int t = 0; t < 2; ++t) {
      sc[t] = f32x4_t(0.f);
      #pragma unroll
      for (int c = 0; c < KC; ++c) sc[t] = mfma16(kf[t][c], qf[c], sc[t]);
    }
    float p[8];
    #pragma unroll
    for (int i = 0; i < 8; ++i) {
      const float w = weigh(sc[i >> 2][i & 3]);
      p[i] = tp + i >= lo && tp + i <= pos ? w : 0.f;
    }
    short8_t ph, pl;
    split_bf16x8(p, &ph, &pl);
    #pragma unroll
    for (int e = 0; e < ET; ++e) {
      acc[e] = mfma16(vf[e], ph, acc[e]);
      acc[e] = mfma16(vf[e], pl, acc[e]);
    }
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
    f32x4_t o = f32x4_t(0.f);
    #pragma unroll
    for (int w = 0; w < 4; ++w)
      o += *reinterpret_cast<const f32x4_t*>(comb + w * n + u);
    const long at = (row * H + h0) * E + u;
    if (split == 1)
      *reinterpret_cast<uint2*>(out + at) =
          uint2{cvt_pk_bf16(o[0], o[1]), cvt_pk_bf16(o[2], o[3])};
    else
      *reinterpret_cast<f32x4_t*>(
          partial + (row * split + z) * (long)H * E + (long)h0 * E + u) = o;
  }
}

// out[row] = sum of the row's parts, n = H * E columns
__global__ __launch_bounds__(256) void sigmoid_attn_merge_kernel(
    bf16* __restrict__ out, const float* __restrict__ partial, int split,
    int n) {
  const int u = (blockIdx.y * 256 + threadIdx.x) * 4;
  if (u >= n) return;
  const float* x = partial + (long)blockIdx.x * split * n + u;
  f32x4_t o = f32x4_t(0.f);
  #pragma unroll 4
  for (int i = 0; i < split; ++i)
    o += *reinterpret_cast<const f32x4_t*>(x + (long)i * n);
  *reinterpret_cast<uint2*>(out + (long)blockIdx.x * n + u) =
      uint2{cvt_pk_bf16(o[0], o[1]), cvt_pk_bf16(o[2], o[3])};
}

}  // namespace

template <typename T>
void launch_sigmoid_attn_general(T* out, const T* q, const T* k_cache,
                                 const T* v_cache, const int* block_tables,
                                 const long* positions, const int* row_seq,
                                 const float* bias, long rows, int max_blocks,
                                 int H, int G, int D, int E, int chunk,
                                 float scale, float cap, long qs,
                                 hipStream_t stream) {
  if (rows == 0) return;
  sigmoid_attn_general_kernel<T>
      <<<dim3((unsigned)rows, (unsigned)H), 256, (D + TILE) * sizeof(float),
         stream>>>(out, q, k_cache, v_cache, block_tables, positions, row_seq,
                   bias, max_blocks, H, G, D, E, chunk, scale, cap, qs);
}
template void launch_sigmoid_attn_general<bf16>(
    bf16*, const bf16*, const bf16*, const bf16*, const int*, const long*,
    const int*, const float*, long, int, int, int, int, int, int, float,
    float, long, hipStream_t);
template void launch_sigmoid_attn_general<float>(
    float*, const float*, const float*, const float*, const int*,
    const long*, const int*, const float*, long, int, int, int, int, int,
    int, float, float, long, hipStream_t);

// padded sizes of the matrix-core kernels
#define SIGMOID_SIZES(CASE)                                                 \
  CASE(64, 64) CASE(64, 128) CASE(128, 128) CASE(64, 256) CASE(128, 256)    \
  CASE(256, 256)

void launch_sigmoid_attn_prefill(bf16* out, const bf16* q,
                                 const bf16* k_cache, const bf16* v_cache,
                                 const int* block_tables,
                                 const long* positions, const int* seq_start,
                                 const int* tiles, const float* bias,
                                 int num_tiles, int max_blocks, int H, int G,
                                 int D, int E, int chunk, float scale,
                                 float cap, long qs, hipStream_t stream) {
  if (num_tiles == 0) return;
  // two heads share a tile's keys where enough workgroups remain
  const int hw = H / G % 2 == 0 && (long)H / 2 * num_tiles >= 512 ? 2 : 1;
  const dim3 grid((unsigned)(H / hw), (unsigned)num_tiles);
  #define RUN(DP, EP, HW)                                                   \
    sigmoid_attn_prefill_kernel<DP, EP, HW><<<grid, 256, 0, stream>>>(      \
        out, q, k_cache, v_cache, block_tables, positions, seq_start,       \
        tiles, bias, max_blocks, H, G, D, E, chunk, scale, cap, qs)
  #define CASE(DP, EP)                                                      \
    if (D <= DP && E <= EP) {                                               \
      if (hw == 2) RUN(DP, EP, 2); else RUN(DP, EP, 1);                     \
      return;                                                               \
    }
  SIGMOID_SIZES(CASE)
  #undef CASE
  #undef RUN
  throw std::runtime_error("sigmoid_attn_prefill: head sizes");
}

void launch_sigmoid_attn_decode(bf16* out, const bf16* q, const bf16* k_cache,
                                const bf16* v_cache, const int* block_tables,
                                const long* positions, const float* bias,
                                float* partial, long rows, int max_blocks,
                                int H, int G, int D, int E, int chunk,
                                float scale, float cap, long qs, int split,
                                hipStream_t stream) {
  if (rows == 0) return;
  const int group = H / G, hb = (group + NC - 1) / NC;
  const int cols = group < NC ? group : NC;
  const size_t lds = (size_t)4 * cols * E * sizeof(float);    // <= 64 KB
  const dim3 grid((unsigned)rows, (unsigned)(G * hb), (unsigned)split);
  #define CASE(DP, EP)                                                      \
    if (D <= DP && E <= EP) {                                               \
      sigmoid_attn_decode_kernel<DP, EP><<<grid, 256, lds, stream>>>(       \
          out, q, k_cache, v_cache, block_tables, positions, bias, partial, \
          max_blocks, H, G, D, E, chunk, scale, cap, qs);                   \
      if (split > 1)                                                        \
        sigmoid_attn_merge_kernel<<<                                        \
            dim3((unsigned)rows, (unsigned)((H * E + 1023) / 1024)), 256,   \
            0, stream>>>(out, partial, split, H * E);                       \
      return;                                                               \
    }
  SIGMOID_SIZES(CASE)
  #undef CASE
  throw std::runtime_error("sigmoid_attn_decode: head sizes");
}
