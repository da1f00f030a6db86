// Inputs of sublayers (gfx950): residual add and norms between two sublayers
// (sublayer.h), and the causal convolution over time that is added to a
// sublayer's input, h_t + sum_j w[j] h_(t - taps + 1 + j) per channel.
//
// A decoded token's convolution happens in the kernel that makes its input.
// In prefill the rows of a portion meet each other: conv_kernel reads the
// finished inputs, ROWS rows and 256 * V columns a workgroup.  Rows before the
// portion come from the sequence's tail [taps - 1, width]; the workgroup of a
// portion's first rows renews it, since no other one reads it (taps - 1 <=
// ROWS; more taps take a kernel of their own for that).
#include "sublayer.h"

namespace {

template <typename T, int V, int NT, bool CONV, int ADD>
__global__ __launch_bounds__(NT) void add_rms_next_kernel(
    Between<T> a, const T* __restrict__ y) {
  const long t = blockIdx.x;
  between_sublayers<T, V, NT, CONV, ADD>(a, t, [&](int c, float* x) {
    load_vec<T, V>(y + t * a.width + c, x);
  });
}

constexpr int TILE = 64;            // rows of a tile of the list
constexpr int ROWS = 4;             // of these per workgroup

template <typename T> struct Conv {
  T* out;
  const T* h;
  const float* w;                   // [taps, width]
  T* tail;
  const int* seq_start;
  const long* positions;
  const int* slots;
  const int* tiles;
  int taps, width;
};

// rows of one portion as the convolution sees them, columns [c, c + V)
template <typename T, int V> struct Rows {
  const T* h;                       // portion's first row
  const T* tail;                    // null: nothing is kept
  long first;                       // position of the first row
  int past, width;

  DEV void load(int r, float* x) const {
    #pragma unroll
    for (int i = 0; i < V; ++i) x[i] = 0.f;
    if (r >= 0)
      load_vec<T, V>(h + (long)r * width, x);
    else if (tail && first + r >= 0)
      load_vec<T, V>(tail + (long)(past + r) * width, x);
  }
};

template <typename T, int V>
DEV Rows<T, V> rows_of(const Conv<T>& a, int s, int c, bool start) {
  const int t0 = a.seq_start[s];
  Rows<T, V> rows{a.h + (long)t0 * a.width + c, nullptr, 0, a.taps - 1,
                  a.width};
  if (start) {
    const int slot = a.slots[s];
    if (slot >= 0) rows.tail = a.tail + (long)slot * rows.past * a.width + c;
    rows.first = a.positions[t0];
  }
  return rows;
}

// the last inputs of a portion of n rows, oldest first: row i is read from
// the tail's row n + i at most, before that one is written
template <typename T, int V>
DEV void renew_tail(const Conv<T>& a, const Rows<T, V>& rows, int s, int n,
                    int c) {
  if (!rows.tail) return;
  T* tail = a.tail + (long)a.slots[s] * rows.past * a.width + c;
  for (int i = 0; i < rows.past; ++i) {
    float x[V];
    rows.load(n - rows.past + i, x);
    store_vec<T, V>(tail + (long)i * a.width, x);
  }
}

// TAPS 0: any number, every row is read again for every tap
template <typename T, int V, int TAPS>
__global__ __launch_bounds__(256) void conv_kernel(Conv<T> a) {
  // neighbouring rows on the same one of the 8 dies: they share past rows
  // through its cache (the grid is a multiple of 8)
  const unsigned b = blockIdx.x % 8 * (gridDim.x / 8) + blockIdx.x / 8;
  const int tile = b / (TILE / ROWS);
  const int s = a.tiles[2 * tile];
  const int r0 = a.tiles[2 * tile + 1] + b % (TILE / ROWS) * ROWS;
  const int n = a.seq_start[s + 1] - a.seq_start[s];
  const int c = (blockIdx.y * 256 + threadIdx.x) * V;
  if (r0 >= n || c >= a.width) return;
  const bool start = r0 < max(a.taps - 1, 1);    // these meet the tail
  const Rows<T, V> rows = rows_of<T, V>(a, s, c, start);
  T* out = a.out + (long)a.seq_start[s] * a.width + c;
  const int r1 = min(r0 + ROWS, n);
  if constexpr (TAPS > 0) {
    float w[TAPS][V], x[ROWS + TAPS - 1][V];
    #pragma unroll
    for (int j = 0; j < TAPS; ++j)
      load_vec<float, V>(a.w + (long)j * a.width + c, w[j]);
    #pragma unroll
    for (int i = 0; i < ROWS + TAPS - 1; ++i) {
      const int r = r0 - (TAPS - 1) + i;
      if (r < r1) rows.load(r, x[i]);
    }
    #pragma unroll
    for (int i = 0; i < ROWS; ++i) {
      if (r0 + i >= r1) break;
      float y[V];
      #pragma unroll
      for (int v = 0; v < V; ++v) {
        y[v] = x[i + TAPS - 1][v];
        #pragma unroll
        for (int j = TAPS - 1; j >= 0; --j) y[v] += w[j][v] * x[i + j][v];
      }
      store_vec<T, V>(out + (long)(r0 + i) * a.width, y);
    }
  } else {
    for (int r = r0; r < r1; ++r) {
      float y[V];
      rows.load(r, y);
      for (int j = a.taps - 1; j >= 0; --j) {
        float w[V], x[V];
        load_vec<float, V>(a.w + (long)j * a.width + c, w);
        rows.load(r - (a.taps - 1) + j, x);
        #pragma unroll
        for (int v = 0; v < V; ++v) y[v] += w[v] * x[v];
      }
      store_vec<T, V>(out + (long)r * a.width, y);
    }
  }
  if (r0 == 0 && a.taps - 1 <= ROWS) renew_tail(a, rows, s, n, c);
}

template <typename T, int V>
__global__ __launch_bounds__(256) void conv_tail_kernel(Conv<T> a) {
  const int s = blockIdx.x, c = (blockIdx.y * 256 + threadIdx.x) * V;
  const int n = a.seq_start[s + 1] - a.seq_start[s];
  if (n <= 0 || c >= a.width) return;
  renew_tail(a, rows_of<T, V>(a, s, c, true), s, n, c);
}

template <typename T, int V>
void run_conv(const Conv<T>& a, int tiles, int seqs, hipStream_t stream) {
  const unsigned cols = (unsigned)((a.width + 256 * V - 1) / (256 * V));
  const dim3 grid((unsigned)tiles * (TILE / ROWS), cols);
  switch (a.taps) {
    case 2: conv_kernel<T, V, 2><<<grid, 256, 0, stream>>>(a); break;
    case 3: conv_kernel<T, V, 3><<<grid, 256, 0, stream>>>(a); break;
    case 4: conv_kernel<T, V, 4><<<grid, 256, 0, stream>>>(a); break;
    default: conv_kernel<T, V, 0><<<grid, 256, 0, stream>>>(a);
  }
  if (a.taps - 1 > ROWS)
    conv_tail_kernel<T, V><<<dim3((unsigned)seqs, cols), 256, 0, stream>>>(a);
}

}  // namespace

template <typename T>
void launch_add_rms_next(const Between<T>& a, const T* y, long rows,
                         hipStream_t stream) {
  if (rows == 0) return;
  #define ADD(V, NT, CONV, HOW)                                             \
    add_rms_next_kernel<T, V, NT, CONV, HOW>                                \
        <<<(unsigned)rows, NT, 0, stream>>>(a, y)
  #define RUN(V, NT, CONV)                                                  \
    if (!y) ADD(V, NT, CONV, ADD_NOTHING);                                  \
    else if (a.post) ADD(V, NT, CONV, ADD_NORMED);                          \
    else ADD(V, NT, CONV, ADD_PLAIN)
  BY_WIDTH(RUN);
  #undef RUN
  #undef ADD
}

template <typename T>
void launch_causal_conv(T* out, const T* h, const float* w, T* tail,
                        const int* seq_start, const long* positions,
                        const int* slots, const int* tiles, int num_tiles,
                        int seqs, int taps, int width, hipStream_t stream) {
  if (num_tiles == 0) return;
  const Conv<T> a{out, h, w, tail, seq_start, positions, slots, tiles, taps,
                  width};
  if (width % 4 == 0)
    run_conv<T, 4>(a, num_tiles, seqs, stream);
  else
    run_conv<T, 1>(a, num_tiles, seqs, stream);
}

#define INSTANTIATE(T)                                                      \
  template void launch_add_rms_next<T>(const Between<T>&, const T*, long,   \
                                       hipStream_t);                        \
  template void launch_causal_conv<T>(                                      \
      T*, const T*, const float*, T*, const int*, const long*, const int*,  \
      const int*, int, int, int, int, hipStream_t);
INSTANTIATE(bf16)
INSTANTIATE(float)
#undef INSTANTIATE
