// An activation that rides along with a kernel of the same rows:
// out = relu(x)^2 for column views x and out [rows, n] of two buffers.  The
// carrying kernel gives it side_blocks(n) workgroups of 256 threads more for
// every group of its rows.
#pragma once

#include "common.h"

template <typename T> struct SideRelu {
  const T* x = nullptr;
  T* out = nullptr;
  long xs = 0, os = 0;      // row strides
  int n = 0;
  bool vec = false;         // 8 columns at a time
};

constexpr int SIDE_COLS = 2048;

inline unsigned side_blocks(int n) {
  return (unsigned)((n + SIDE_COLS - 1) / SIDE_COLS);
}

// 8 columns at a time want sizes, strides and bases in multiples of 8
template <typename T>
SideRelu<T> make_side(const T* x, T* out, long xs, long os, int n) {
  auto aligned = [](const T* p) {
    return reinterpret_cast<uintptr_t>(p) % (8 * sizeof(T)) == 0;
  };
  return {x, out, xs, os, n, n % 8 == 0 && xs % 8 == 0 && os % 8 == 0 &&
                                 aligned(x) && aligned(out)};
}

template <typename T>
DEV void side_relu(const SideRelu<T>& s, long row0, int rows, int block) {
  const int c0 = block * SIDE_COLS;
  if (s.vec) {
    const int c = c0 + threadIdx.x * 8;
    if (c >= s.n) return;
    #pragma unroll 4
    for (int r = 0; r < rows; ++r) {
      float f[8];
      load_vec<T, 8>(s.x + (row0 + r) * s.xs + c, f);
      #pragma unroll
      for (int i = 0; i < 8; ++i) {
        f[i] = fmaxf(f[i], 0.f);
        f[i] *= f[i];
      }
      store_vec<T, 8>(s.out + (row0 + r) * s.os + c, f);
    }
    return;
  }
  const int c1 = min(c0 + SIDE_COLS, s.n);
  for (int r = 0; r < rows; ++r)
    for (int c = c0 + threadIdx.x; c < c1; c += 256) {
      const float f = fmaxf(Elem<T>::ld(s.x + (row0 + r) * s.xs + c), 0.f);
      Elem<T>::st(s.out + (row0 + r) * s.os + c, f * f);
    }
}
