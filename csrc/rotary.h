// Cosine and sine of position * frequency, frequencies in double: the angle is
// reduced in double, so it stays exact to float rounding at any position.
#pragma once

#include "common.h"

// T: element type of the kernel.  16-bit kernels take the hardware functions,
// whose argument is in turns.
template <typename T>
DEV void angle(long position, double freq, float* c, float* s) {
  // in turns, reduced to [-1/2, 1/2]
  double a = (double)position * freq * 0.15915494309189535;
  a -= rint(a);
  if constexpr (sizeof(T) == 2) {
    *s = __builtin_amdgcn_sinf((float)a);
    *c = __builtin_amdgcn_cosf((float)a);
  } else {
    sincosf((float)(a * 6.283185307179586), s, c);
  }
}

// x[2i], x[2i + 1] turned by (cos, sin) pairs cs
template <int N> DEV void turn_pairs(float* x, const float* cs) {
  #pragma unroll
  for (int i = 0; i < N; i += 2) {
    const float c = cs[i], s = cs[i + 1], u = x[i], v = x[i + 1];
    x[i] = u * c - v * s;
    x[i + 1] = v * c + u * s;
  }
}
