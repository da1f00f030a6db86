// RMS norms around a float residual stream (gfx950): scaled embedding, norm
// of the residual, norm-and-add of a sublayer's output, the norm and sigmoid
// gate over all heads of a linear-attention layer, and the gated GELU against
// a token's own table entry.
//
// One 256-thread workgroup a row.  The residual and the norm weights are
// float; sublayer outputs have the model's element type T.  Rows of up to
// 256 * V * HELD elements stay in registers between the two passes, longer
// ones are read again.
#include "common.h"

namespace {

constexpr int HELD = 4;

// sum of squares, then use(c, x): x[V] at column c
template <typename T, int V, typename Use>
DEV void rms_row(const T* x, int n, float* scratch, float eps, float ss_all,
                 float count, Use use) {
  const int tid = threadIdx.x;
  float held[HELD][V];
  float ss = 0.f;
  #pragma unroll
  for (int i = 0; i < HELD; ++i) {
    const int c = (i * 256 + tid) * V;
    if (c < n) {
      load_vec<T, V>(x + c, held[i]);
      #pragma unroll
      for (int j = 0; j < V; ++j) ss += held[i][j] * held[i][j];
    }
  }
  for (int c = (HELD * 256 + tid) * V; c < n; c += 256 * V) {
    float f[V];
    load_vec<T, V>(x + c, f);
    #pragma unroll
    for (int j = 0; j < V; ++j) ss += f[j] * f[j];
  }
  if (ss_all < 0.f)
    ss = block_reduce_sum_256(ss, scratch);
  else
    ss = ss_all;
  const float rs = 1.f / sqrtf(ss / count + eps);
  #pragma unroll
  for (int i = 0; i < HELD; ++i) {
    const int c = (i * 256 + tid) * V;
    if (c < n) {
      #pragma unroll
      for (int j = 0; j < V; ++j) held[i][j] *= rs;
      use(c, held[i]);
    }
  }
  for (int c = (HELD * 256 + tid) * V; c < n; c += 256 * V) {
    float f[V];
    load_vec<T, V>(x + c, f);
    #pragma unroll
    for (int j = 0; j < V; ++j) f[j] *= rs;
    use(c, f);
  }
}

// residual[t] = table[ids[t]] * scale; out[t] the same (null: none)
template <typename T, int V>
__global__ __launch_bounds__(256) void embed_scaled_kernel(
    T* __restrict__ out, float* __restrict__ residual,
    const T* __restrict__ table, const long* __restrict__ ids, float scale,
    int width, long vocab) {
  const long row = blockIdx.x;
  const int c = (blockIdx.y * 256 + threadIdx.x) * V;
  if (c >= width) return;
  long id = ids[row];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  float x[V];
  load_vec<T, V>(table + id * width + c, x);
  #pragma unroll
  for (int i = 0; i < V; ++i) x[i] *= scale;
  store_vec<float, V>(residual + row * width + c, x);
  if (out) store_vec<T, V>(out + row * width + c, x);
}

template <typename T, int V>
__global__ __launch_bounds__(256) void rms_scale_kernel(
    T* __restrict__ out, const float* __restrict__ x,
    const float* __restrict__ w, int width, float eps) {
  __shared__ float scratch[4];
  const long at = (long)blockIdx.x * width;
  rms_row<float, V>(x + at, width, scratch, eps, -1.f, width,
                    [&](int c, float* f) {
    float wv[V];
    load_vec<float, V>(w + c, wv);
    #pragma unroll
    for (int i = 0; i < V; ++i) f[i] *= wv[i];
    store_vec<T, V>(out + at + c, f);
  });
}

// residual += rms(h) * w; out = the residual (null: none)
template <typename T, int V>
__global__ __launch_bounds__(256) void add_rms_kernel(
    T* __restrict__ out, float* __restrict__ residual,
    const T* __restrict__ h, const float* __restrict__ w, int width,
    float eps) {
  __shared__ float scratch[4];
  const long at = (long)blockIdx.x * width;
  rms_row<T, V>(h + at, width, scratch, eps, -1.f, width,
                [&](int c, float* f) {
    float wv[V], r[V];
    load_vec<float, V>(w + c, wv);
    load_vec<float, V>(residual + at + c, r);
    #pragma unroll
    for (int i = 0; i < V; ++i) r[i] += f[i] * wv[i];
    store_vec<float, V>(residual + at + c, r);
    if (out) store_vec<T, V>(out + at + c, r);
  });
}

// y = rms(o) * w * sigmoid(g); with ss the row's sum of squares over `total`
// columns comes from there (o holds only part of them)
template <typename T, int V>
__global__ __launch_bounds__(256) void rms_gate_kernel(
    T* __restrict__ y, const float* __restrict__ o, const T* __restrict__ g,
    const float* __restrict__ w, const float* __restrict__ ss, int n,
    long total, long stride, float eps) {
  __shared__ float scratch[4];
  const long row = blockIdx.x, at = row * n;
  rms_row<float, V>(o + at, n, scratch, eps, ss ? ss[row] : -1.f,
                    (float)total, [&](int c, float* f) {
    float wv[V], gv[V];
    load_vec<float, V>(w + c, wv);
    load_vec<T, V>(g + row * stride + c, gv);
    #pragma unroll
    for (int i = 0; i < V; ++i)
      f[i] *= wv[i] / (1.f + Fn<T>::exp(-gv[i]));
    store_vec<T, V>(y + at + c, f);
  });
}

// ss[t] = sum of squares of row t
__global__ __launch_bounds__(256) void row_squares_kernel(
    float* __restrict__ ss, const float* __restrict__ x, int n) {
  __shared__ float scratch[4];
  const float* row = x + (long)blockIdx.x * n;
  float s = 0.f;
  for (int c = threadIdx.x; c < n; c += 256) s += row[c] * row[c];
  s = block_reduce_sum_256(s, scratch);
  if (threadIdx.x == 0) ss[blockIdx.x] = s;
}

// out[t, j] = gelu_tanh(z[t, j]) * table[ids[t], column + j]
template <typename T, int V>
__global__ __launch_bounds__(256) void gelu_gate_kernel(
    T* __restrict__ out, const T* __restrict__ z, const T* __restrict__ table,
    const long* __restrict__ ids, long rows, int n, long cols, long column,
    long vocab) {
  const int units = n / V;
  const long u = (long)blockIdx.x * 256 + threadIdx.x;
  const long row = u / units;
  if (row >= rows) return;
  const int j = (int)(u - row * units) * V;
  long id = ids[row];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  float v[V], e[V];
  load_vec<T, V>(z + row * n + j, v);
  load_vec<T, V>(table + id * cols + column + j, e);
  #pragma unroll
  for (int i = 0; i < V; ++i) {
    const float s = 0.7978845608028654f *
                    (v[i] + 0.044715f * v[i] * v[i] * v[i]);
    v[i] = 0.5f * v[i] * (1.f + Fn<T>::tanh(s)) * e[i];
  }
  store_vec<T, V>(out + row * n + j, v);
}

bool by4(const void* p, size_t elem) {
  return reinterpret_cast<uintptr_t>(p) % (4 * elem) == 0;
}

}  // namespace

template <typename T>
void launch_embed_scaled(T* out, float* residual, const T* table,
                         const long* ids, float scale, long rows, int width,
                         long vocab, hipStream_t stream) {
  if (rows == 0) return;
  if (width % 4 == 0)
    embed_scaled_kernel<T, 4>
        <<<dim3((unsigned)rows, (unsigned)((width / 4 + 255) / 256)), 256, 0,
           stream>>>(out, residual, table, ids, scale, width, vocab);
  else
    embed_scaled_kernel<T, 1>
        <<<dim3((unsigned)rows, (unsigned)((width + 255) / 256)), 256, 0,
           stream>>>(out, residual, table, ids, scale, width, vocab);
}

template <typename T>
void launch_rms_scale(T* out, const float* x, const float* w, long rows,
                      int width, float eps, hipStream_t stream) {
  if (rows == 0) return;
  if (width % 4 == 0)
    rms_scale_kernel<T, 4><<<(unsigned)rows, 256, 0, stream>>>(out, x, w,
                                                               width, eps);
  else
    rms_scale_kernel<T, 1><<<(unsigned)rows, 256, 0, stream>>>(out, x, w,
                                                               width, eps);
}

template <typename T>
void launch_add_rms(T* out, float* residual, const T* h, const float* w,
                    long rows, int width, float eps, hipStream_t stream) {
  if (rows == 0) return;
  if (width % 4 == 0)
    add_rms_kernel<T, 4><<<(unsigned)rows, 256, 0, stream>>>(
        out, residual, h, w, width, eps);
  else
    add_rms_kernel<T, 1><<<(unsigned)rows, 256, 0, stream>>>(
        out, residual, h, w, width, eps);
}

template <typename T>
void launch_rms_gate(T* y, const float* o, const T* g, const float* w,
                     const float* ss, long rows, int n, long total,
                     long stride, float eps, hipStream_t stream) {
  if (rows == 0) return;
  if (n % 4 == 0 && stride % 4 == 0 && by4(g, sizeof(T)))
    rms_gate_kernel<T, 4><<<(unsigned)rows, 256, 0, stream>>>(
        y, o, g, w, ss, n, total, stride, eps);
  else
    rms_gate_kernel<T, 1><<<(unsigned)rows, 256, 0, stream>>>(
        y, o, g, w, ss, n, total, stride, eps);
}

void launch_row_squares(float* ss, const float* x, long rows, int n,
                        hipStream_t stream) {
  if (rows == 0) return;
  row_squares_kernel<<<(unsigned)rows, 256, 0, stream>>>(ss, x, n);
}

template <typename T>
void launch_gelu_gate(T* out, const T* z, const T* table, const long* ids,
                      long rows, int n, long cols, long column, long vocab,
                      hipStream_t stream) {
  if (rows == 0 || n == 0) return;
  if (n % 4 == 0 && cols % 4 == 0 && column % 4 == 0)
    gelu_gate_kernel<T, 4>
        <<<(unsigned)((rows * (n / 4) + 255) / 256), 256, 0, stream>>>(
            out, z, table, ids, rows, n, cols, column, vocab);
  else
    gelu_gate_kernel<T, 1>
        <<<(unsigned)((rows * n + 255) / 256), 256, 0, stream>>>(
            out, z, table, ids, rows, n, cols, column, vocab);
}

#define INSTANTIATE(T)                                                      \
  template void launch_embed_scaled<T>(T*, float*, const T*, const long*,   \
                                       float, long, int, long,              \
                                       hipStream_t);                        \
  template void launch_rms_scale<T>(T*, const float*, const float*, long,   \
                                    int, float, hipStream_t);               \
  template void launch_add_rms<T>(T*, float*, const T*, const float*, long, \
                                  int, float, hipStream_t);                 \
  template void launch_rms_gate<T>(T*, const float*, const T*,              \
                                   const float*, const float*, long, int,   \
                                   long, long, float, hipStream_t);         \
  template void launch_gelu_gate<T>(T*, const T*, const T*, const long*,    \
                                    long, int, long, long, long,            \
                                    hipStream_t);
INSTANTIATE(bf16)
INSTANTIATE(float)
#undef INSTANTIATE
