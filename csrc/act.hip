// Fused SwiGLU: out[t, i] = silu(x[t, i]) * x[t, I + i] — one pass,
// bf16x8-vectorized.  Row-indexed 2-D grid: the flat grid-stride form
// spent a 64-bit div/mod per 16 B on address math and measured 4x off
// the HBM stream floor at the MoE shape (172 us vs ~44 us for 352 MB).
#include "common.h"

// CLAMPED: the clamped unit instead of silu(gate) * up
template <bool CLAMPED>
__global__ __launch_bounds__(256) void silu_mul_kernel(
    bf16* __restrict__ out, const bf16* __restrict__ x, long rows,
    int inter, float limit) {
  const long t = blockIdx.y;
  const int nv = inter / 8;
  const bf16* row = x + t * 2 * (long)inter;
  bf16* orow = out + t * (long)inter;
  for (int v = blockIdx.x * 256 + threadIdx.x; v < nv;
       v += gridDim.x * 256) {
    const int j = v * 8;
    bf16x8 g = load_bf16x8(row + j);
    bf16x8 p = load_bf16x8(row + inter + j);
    bf16x8 o;
    #pragma unroll
    for (int i = 0; i < 8; ++i) {
      const float gv = bf16x8_get(g, i);
      if constexpr (CLAMPED) {
        bf16x8_set(o, i, clamped_unit<bf16>(gv, bf16x8_get(p, i), limit));
      } else {
        const float s = gv / (1.f + __expf(-gv));
        bf16x8_set(o, i, s * bf16x8_get(p, i));
      }
    }
    store_bf16x8(orow + j, o);
  }
}

template <bool CLAMPED>
static void run_silu_mul(bf16* out, const bf16* x, long rows, int inter,
                         float limit, hipStream_t stream) {
  const int nv = inter / 8;
  // fill the chip but bound blocks-per-row; rows beyond 65535 (grid.y
  // limit) take a strided outer pass
  const unsigned bx = (unsigned)min((nv + 255) / 256, 32);
  for (long r0 = 0; r0 < rows; r0 += 65535) {
    const long nr = min(rows - r0, (long)65535);
    silu_mul_kernel<CLAMPED><<<dim3(bx, (unsigned)nr), 256, 0, stream>>>(
        out + r0 * inter, x + r0 * 2 * (long)inter, nr, inter, limit);
  }
}

void launch_silu_mul(bf16* out, const bf16* x, long rows, int inter,
                     hipStream_t stream) {
  run_silu_mul<false>(out, x, rows, inter, 0.f, stream);
}

template <typename T>
__global__ __launch_bounds__(256) void clamped_glu_kernel(
    T* __restrict__ out, const T* __restrict__ x, int inter, float limit) {
  const long t = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c < inter)
    Elem<T>::st(out + t * inter + c,
                clamped_unit<T>(Elem<T>::ld(x + t * 2 * inter + c),
                                Elem<T>::ld(x + t * 2 * inter + inter + c),
                                limit));
}

// element type bf16 or float, any inner size
template <typename T>
void launch_clamped_glu(T* out, const T* x, long rows, int inter, float limit,
                        hipStream_t stream) {
  if (rows == 0) return;
  if constexpr (sizeof(T) == 2)
    if (inter % 8 == 0)
      return run_silu_mul<true>(out, x, rows, inter, limit, stream);
  clamped_glu_kernel<T><<<dim3((unsigned)rows,
                               (unsigned)((inter + 255) / 256)),
                          256, 0, stream>>>(out, x, inter, limit);
}
template void launch_clamped_glu<bf16>(bf16*, const bf16*, long, int, float,
                                       hipStream_t);
template void launch_clamped_glu<float>(float*, const float*, long, int,
                                        float, hipStream_t);

// x = relu(x)^2 in place, V elements (16 bytes, or one) a thread
template <typename T, int V>
__global__ __launch_bounds__(256) void squared_relu_kernel(T* __restrict__ x,
                                                           long n) {
  const long i = ((long)blockIdx.x * 256 + threadIdx.x) * V;
  if (i >= n) return;
  float f[V];
  #pragma unroll
  for (int j = 0; j < V; j += V == 1 ? 1 : 4)
    load_vec<T, V == 1 ? 1 : 4>(x + i + j, f + j);
  #pragma unroll
  for (int j = 0; j < V; ++j) {
    const float r = fmaxf(f[j], 0.f);
    f[j] = r * r;
  }
  #pragma unroll
  for (int j = 0; j < V; j += V == 1 ? 1 : 4)
    store_vec<T, V == 1 ? 1 : 4>(x + i + j, f + j);
}

template <typename T>
void launch_squared_relu(T* x, long n, hipStream_t stream) {
  constexpr int V = 16 / sizeof(T);
  if (n == 0) return;
  if (n % V == 0)
    squared_relu_kernel<T, V><<<(unsigned)((n / V + 255) / 256), 256, 0,
                                stream>>>(x, n);
  else
    squared_relu_kernel<T, 1><<<(unsigned)((n + 255) / 256), 256, 0,
                                stream>>>(x, n);
}
template void launch_squared_relu<bf16>(bf16*, long, hipStream_t);
template void launch_squared_relu<float>(float*, long, hipStream_t);

// Fused gated GELU (tanh form): out[t, i] = gelu(x[t, i]) * x[t, I + i],
// element type bf16 or float, any inner size.
template <typename T, int V>
__global__ __launch_bounds__(256) void gelu_mul_kernel(
    T* __restrict__ out, const T* __restrict__ x, int inter) {
  const long t = blockIdx.x;
  const int c = (blockIdx.y * 256 + threadIdx.x) * V;
  if (c >= inter) return;
  float g[V], u[V];
  load_vec<T, V>(x + t * 2 * inter + c, g);
  load_vec<T, V>(x + t * 2 * inter + inter + c, u);
  #pragma unroll
  for (int i = 0; i < V; ++i) {
    const float z = g[i];
    const float s = 0.7978845608028654f * (z + 0.044715f * z * z * z);
    g[i] = 0.5f * z * (1.f + Fn<T>::tanh(s)) * u[i];
  }
  store_vec<T, V>(out + t * inter + c, g);
}

template <typename T>
void launch_gelu_mul(T* out, const T* x, long rows, int inter,
                     hipStream_t stream) {
  if (rows == 0) return;
  if (inter % 4 == 0)          // 4 elements a thread
    gelu_mul_kernel<T, 4><<<dim3((unsigned)rows,
                                 (unsigned)((inter / 4 + 255) / 256)),
                            256, 0, stream>>>(out, x, inter);
  else
    gelu_mul_kernel<T, 1><<<dim3((unsigned)rows,
                                 (unsigned)((inter + 255) / 256)),
                            256, 0, stream>>>(out, x, inter);
}
template void launch_gelu_mul<bf16>(bf16*, const bf16*, long, int,
                                    hipStream_t);
template void launch_gelu_mul<float>(float*, const float*, long, int,
                                     hipStream_t);
