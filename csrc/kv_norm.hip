// RMS norm of query and key heads, and paged append without rotation (gfx950).
//
//   q [T, H * D]  normed in place     k [T, G * D]  normed into the page
//   v [T, G * E]                      weights [D] float, shared by all heads
//   k_cache [NB, G, BS, D]            v_cache [NB, G, E, BS]
//
// V elements a lane at a time (1 or 8; 8 wants D, E, strides and bases in
// multiples of 8); a power of two of lanes has a head.  A workgroup takes TB
// neighbouring rows, blockIdx.y their q (0) or their k and v (1).  With TB > 1
// tokens run fastest over the lanes of a V store, so the transposed writes of
// one sequence meet in the same page rows.
#include "common.h"

namespace {

// one head by `lanes` lanes (this one is `l`); dst may be x
template <typename T, int V>
DEV void norm_head(T* dst, const T* x, const float* w, int D, int l,
                   int lanes, float eps) {
  float ss = 0.f;
  for (int d = l * V; d < D; d += lanes * V) {
    float f[V];
    load_vec<T, V>(x + d, f);
    #pragma unroll
    for (int i = 0; i < V; ++i) ss += f[i] * f[i];
  }
  for (int o = lanes >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o);
  const float rs = 1.f / sqrtf(ss / D + eps);
  for (int d = l * V; d < D; d += lanes * V) {
    float f[V], g[V];
    load_vec<T, V>(x + d, f);
    load_vec<float, V>(w + d, g);
    #pragma unroll
    for (int i = 0; i < V; ++i) f[i] *= rs * g[i];
    if (dst) store_vec<T, V>(dst + d, f);
  }
}

template <typename T, int V, int TB>
__global__ __launch_bounds__(256) void norm_append_kernel(
    T* __restrict__ q, const T* __restrict__ k, const T* __restrict__ v,
    const float* __restrict__ qw, const float* __restrict__ kw,
    const long* __restrict__ slot_mapping, T* __restrict__ k_cache,
    T* __restrict__ v_cache, int H, int G, int D, int E, int block_size,
    int lanes, long qs, long ks, long vs, long rows, float eps) {
  __shared__ long slot_of[TB];
  const long row0 = (long)blockIdx.x * TB;
  const int nrows = (int)min((long)TB, rows - row0);
  const int l = threadIdx.x & (lanes - 1), unit = threadIdx.x / lanes;
  const int units = 256 / lanes;
  if (blockIdx.y == 0) {
    for (int u = unit; u < nrows * H; u += units) {
      T* x = q + (row0 + u / H) * qs + (long)(u % H) * D;
      norm_head<T, V>(x, x, qw, D, l, lanes, eps);
    }
    return;
  }
  if (threadIdx.x < nrows)
    slot_of[threadIdx.x] = slot_mapping[row0 + threadIdx.x];
  __syncthreads();
  for (int u = unit; u < nrows * G; u += units) {
    const int b = u / G, g = u % G;
    const long slot = slot_of[b];
    T* dst = slot < 0 ? nullptr
        : k_cache + ((slot / block_size * G + g) * block_size +
                     slot % block_size) * D;
    norm_head<T, V>(dst, k + (row0 + b) * ks + (long)g * D, kw, D, l, lanes,
                    eps);
  }
  for (int u = threadIdx.x; u < TB * (G * E / V); u += 256) {
    const int b = u % TB, c = u / TB * V;
    if (b >= nrows || slot_of[b] < 0) continue;
    const long blk = slot_of[b] / block_size, off = slot_of[b] % block_size;
    T* dst = v_cache + (blk * G * E + c) * block_size + off;
    float x[V];
    load_vec<T, V>(v + (row0 + b) * vs + c, x);
    #pragma unroll
    for (int i = 0; i < V; ++i) Elem<T>::st(dst + (long)i * block_size, x[i]);
  }
}

}  // namespace

template <typename T>
void launch_norm_append(T* q, const T* k, const T* v, const float* qw,
                        const float* kw, const long* slot_mapping, T* k_cache,
                        T* v_cache, long rows, int H, int G, int D, int E,
                        int block_size, long qs, long ks, long vs, float eps,
                        hipStream_t stream) {
  if (rows == 0) return;
  auto aligned = [](const T* p) {
    return reinterpret_cast<uintptr_t>(p) % (8 * sizeof(T)) == 0;
  };
  const bool vec = D % 8 == 0 && E % 8 == 0 && qs % 8 == 0 && ks % 8 == 0 &&
                   vs % 8 == 0 && aligned(q) && aligned(k) && aligned(v);
  int lanes = 1;
  while (lanes < 64 && lanes * (vec ? 8 : 1) < D) lanes *= 2;
  #define RUN(V, TB)                                                        \
    norm_append_kernel<T, V, TB>                                            \
        <<<dim3((unsigned)((rows + TB - 1) / TB), 2), 256, 0, stream>>>(    \
            q, k, v, qw, kw, slot_mapping, k_cache, v_cache, H, G, D, E,    \
            block_size, lanes, qs, ks, vs, rows, eps)
  if (!vec)
    RUN(1, 1);
  else if (rows >= 4096)
    RUN(8, 8);
  else if (rows >= 1024)
    RUN(8, 4);
  else
    RUN(8, 1);
  #undef RUN
}

#define INSTANTIATE(T)                                                      \
  template void launch_norm_append<T>(                                      \
      T*, const T*, const T*, const float*, const float*, const long*, T*,  \
      T*, long, int, int, int, int, int, long, long, long, float,           \
      hipStream_t);
INSTANTIATE(bf16)
INSTANTIATE(float)
#undef INSTANTIATE
