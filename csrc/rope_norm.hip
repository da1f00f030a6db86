// Rotation and RMS norm of query and key heads, rotation of values, paged
// append (gfx950).
//
//   q [T, H * D]  in place            k [T, G * D]  into the page
//   v [T, G * E]                      k_cache [NB, G, BS, D]
//                                     v_cache [NB, G, E, BS]
//
// Neighbouring dimensions are a pair.  The first `rot` dimensions of a q or k
// head turn by position * freqs[i]; with `norm` the head is then divided by
// its root mean square.  The first `vrot` (all, or none) dimensions of a value
// turn by position * turn[i].
//
// A lane has W = max(V, 2) elements at a time (V = 8 wants D, E, strides and
// bases in multiples of 8); a power of two of lanes has a head.  A workgroup
// takes TB neighbouring rows; blockIdx.y 0 has their q, 1 their k and v, the
// others an activation of the same rows.  With TB > 1 tokens run fastest over
// the lanes of a V store, so the transposed writes of one sequence meet in the
// same page rows.
#include <algorithm>

#include "rotary.h"
#include "side.h"

namespace {

template <typename T> struct RopeNorm {
  T* q;
  const T* k;
  const T* v;
  const long* positions;
  const double* freqs;
  const double* turn;
  const long* slot_mapping;
  T* k_cache;
  T* v_cache;
  long rows, qs, ks, vs;
  int H, G, D, E, rot, vrot, block_size, lanes;
  float gain, eps;
  bool norm;
  SideRelu<T> side;
};

// `n` elements of a row of `size`, from d on; single elements one by one
template <typename T, int V, int W>
DEV void load_part(const T* p, int d, int size, float* x) {
  if constexpr (V > 1) {
    load_vec<T, V>(p + d, x);
  } else {
    #pragma unroll
    for (int i = 0; i < W; ++i)
      x[i] = d + i < size ? Elem<T>::ld(p + d + i) : 0.f;
  }
}
template <typename T, int V, int W>
DEV void store_part(T* p, int d, int size, const float* x) {
  if constexpr (V > 1) {
    store_vec<T, V>(p + d, x);
  } else {
    #pragma unroll
    for (int i = 0; i < W; ++i)
      if (d + i < size) Elem<T>::st(p + d + i, x[i]);
  }
}

template <int W> DEV void turn_part(float* x, int d, int rot,
                                    const float* cs) {
  #pragma unroll
  for (int i = 0; i < W; i += 2)
    if (d + i < rot) turn_pairs<2>(x + i, cs + d + i);
}

// one head by a.lanes lanes, this one is `l`; dst may be x, null: no store
template <typename T, int V>
DEV void rope_norm_head(const RopeNorm<T>& a, T* dst, const T* x,
                        const float* cs, int l) {
  constexpr int W = V == 1 ? 2 : V;
  const int d0 = l * W, step = a.lanes * W;
  float x0[W], ss = 0.f;
  auto get = [&](int d, float* f) {
    load_part<T, V, W>(x, d, a.D, f);
    turn_part<W>(f, d, a.rot, cs);
  };
  auto squares = [&](const float* f) {
    #pragma unroll
    for (int i = 0; i < W; ++i) ss += f[i] * f[i];
  };
  if (d0 < a.D) {
    get(d0, x0);
    squares(x0);
  }
  if (a.norm)
    for (int d = d0 + step; d < a.D; d += step) {
      float f[W];
      get(d, f);
      squares(f);
    }
  for (int o = a.lanes >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o);
  const float rs = a.norm ? 1.f / sqrtf(ss / a.D + a.eps) : 1.f;
  if (!dst) return;
  for (int d = d0; d < a.D; d += step) {
    float f[W];
    if (d > d0) get(d, f);
    #pragma unroll
    for (int i = 0; i < W; ++i) f[i] = (d > d0 ? f[i] : x0[i]) * rs;
    store_part<T, V, W>(dst, d, a.D, f);
  }
}

template <typename T, int V, int TB>
__global__ __launch_bounds__(256) void rope_norm_append_kernel(
    RopeNorm<T> a) {
  extern __shared__ float cs_all[];    // [TB][rot + vrot] (cos, sin)
  __shared__ long slot_of[TB];
  constexpr int W = V == 1 ? 2 : V;
  const long row0 = (long)blockIdx.x * TB;
  const int nrows = (int)min((long)TB, a.rows - row0);
  if (blockIdx.y >= 2) {
    side_relu(a.side, row0, nrows, blockIdx.y - 2);
    return;
  }
  const bool queries = blockIdx.y == 0;
  const int width = a.rot + a.vrot;
  const int pairs = (queries ? a.rot : width) / 2;
  if (!queries && threadIdx.x < nrows)
    slot_of[threadIdx.x] = a.slot_mapping[row0 + threadIdx.x];
  for (int u = threadIdx.x; u < nrows * pairs; u += 256) {
    const int b = u / pairs, i = u % pairs;
    const bool key = 2 * i < a.rot;
    float c, s;
    angle<T>(a.positions[row0 + b],
             key ? a.freqs[i] : a.turn[i - a.rot / 2], &c, &s);
    const float g = key ? a.gain : 1.f;
    cs_all[b * width + 2 * i] = c * g;
    cs_all[b * width + 2 * i + 1] = s * g;
  }
  __syncthreads();
  // every lane of a head's group takes the same trips: a group is a unit
  const int l = threadIdx.x & (a.lanes - 1), unit = threadIdx.x / a.lanes;
  const int units = 256 / a.lanes;
  if (queries) {
    for (int u = unit; u < nrows * a.H; u += units) {
      T* x = a.q + (row0 + u / a.H) * a.qs + (long)(u % a.H) * a.D;
      rope_norm_head<T, V>(a, x, x, cs_all + u / a.H * width, l);
    }
    return;
  }
  for (int u = unit; u < nrows * a.G; u += units) {
    const int b = u / a.G, g = u % a.G;
    const long slot = slot_of[b];
    T* dst = slot < 0 ? nullptr
        : a.k_cache + ((slot / a.block_size * a.G + g) * a.block_size +
                       slot % a.block_size) * a.D;
    rope_norm_head<T, V>(a, dst, a.k + (row0 + b) * a.ks + (long)g * a.D,
                         cs_all + b * width, l);
  }
  const int per = (a.E + W - 1) / W;             // parts of a value
  for (int u = threadIdx.x; u < TB * a.G * per; u += 256) {
    const int b = u % TB, g = u / TB / per, d = u / TB % per * W;
    if (b >= nrows || slot_of[b] < 0) continue;
    const long blk = slot_of[b] / a.block_size, off = slot_of[b] % a.block_size;
    float x[W];
    load_part<T, V, W>(a.v + (row0 + b) * a.vs + (long)g * a.E, d, a.E, x);
    turn_part<W>(x, d, a.vrot, cs_all + b * width + a.rot);
    T* dst = a.v_cache + ((blk * a.G + g) * a.E + d) * a.block_size + off;
    #pragma unroll
    for (int i = 0; i < W; ++i)
      if (V > 1 || d + i < a.E)
        Elem<T>::st(dst + (long)i * a.block_size, x[i]);
  }
}

}  // namespace

template <typename T>
void launch_rope_norm_append(T* q, const T* k, const T* v,
                             const long* positions, const double* freqs,
                             const double* turn, const long* slot_mapping,
                             T* k_cache, T* v_cache, long rows, int H, int G,
                             int D, int E, int rot, int vrot, int block_size,
                             long qs, long ks, long vs, float gain, float eps,
                             bool norm, const SideRelu<T>& side,
                             hipStream_t stream) {
  if (rows == 0) return;
  auto aligned = [](const T* p) {
    return reinterpret_cast<uintptr_t>(p) % (8 * sizeof(T)) == 0;
  };
  const bool vec = D % 8 == 0 && E % 8 == 0 && qs % 8 == 0 && ks % 8 == 0 &&
                   vs % 8 == 0 && aligned(q) && aligned(k) && aligned(v);
  int lanes = 1;
  while (lanes < 64 && lanes * (vec ? 8 : 2) < D) lanes *= 2;
  const RopeNorm<T> a{q, k, v, positions, freqs, turn, slot_mapping, k_cache,
                      v_cache, rows, qs, ks, vs, H, G, D, E, rot, vrot,
                      block_size, lanes, gain, eps, norm, side};
  #define RUN(V, TB)                                                        \
    rope_norm_append_kernel<T, V, TB>                                       \
        <<<dim3((unsigned)((rows + TB - 1) / TB), 2 + side_blocks(side.n)), \
           256, (TB * (rot + vrot) + 2) * sizeof(float), stream>>>(a)
  if (!vec)
    RUN(1, 1);
  else if (rows >= 4096 && rot + vrot <= 1024)
    RUN(8, 8);
  else if (rows >= 1024 && rot + vrot <= 1024)
    RUN(8, 4);
  else
    RUN(8, 1);
  #undef RUN
}

#define INSTANTIATE(T)                                                      \
  template void launch_rope_norm_append<T>(                                 \
      T*, const T*, const T*, const long*, const double*, const double*,    \
      const long*, T*, T*, long, int, int, int, int, int, int, int, long,   \
      long, long, float, float, bool, const SideRelu<T>&, hipStream_t);
INSTANTIATE(bf16)
INSTANTIATE(float)
#undef INSTANTIATE
