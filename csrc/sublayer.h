// Between two sublayers, one row by a 256-thread workgroup:
//
//   residual += rms(y) * post          (not before the first sublayer)
//   h = rms(residual) * pre, rounded to T
//   out = h, or for a decoded token h + sum_j conv[j] * (input taps-1-j ago)
//
// y comes from value(c, y[V]), columns [c, c + V).  The residual and the norm
// and convolution weights are float.  The inputs that the convolution looks
// back at are kept in tail[slot], oldest first; those from before position 0
// count as zero whatever the slot holds.  Rows of up to 256 * V * HELD columns
// stay in registers.
#pragma once

#include "common.h"

template <typename T> struct Between {
  T* out;
  float* residual;
  const float* post;
  const float* pre;
  const float* conv;        // [taps, width], null: no convolution here
  T* tail;                  // [slots, taps - 1, width]
  const int* slots;         // [rows], -1: nothing is kept
  const long* positions;    // [rows]
  int taps, width;
  float eps;
};

// f as it reads back after a store to T
template <typename T> DEV float as_elem(float f) {
  if constexpr (sizeof(T) == 2) return bf2f(f2bf(f));
  else return f;
}

template <typename T, int V>
DEV void store_input(const Between<T>& a, long t, int c, float* h) {
  T* out = a.out + t * a.width + c;
  if (!a.conv) {
    store_vec<T, V>(out, h);
    return;
  }
  const int past = a.taps - 1, slot = a.slots[t];
  const long p = a.positions[t];
  T* tail = a.tail + (long)slot * past * a.width + c;
  float w[V], y[V];
  load_vec<float, V>(a.conv + (long)past * a.width + c, w);
  #pragma unroll
  for (int i = 0; i < V; ++i) {
    h[i] = as_elem<T>(h[i]);
    y[i] = h[i] + w[i] * h[i];
  }
  for (int j = 0; j < past; ++j) {
    float x[V] = {};
    if (slot >= 0 && p - past + j >= 0)
      load_vec<T, V>(tail + (long)j * a.width, x);
    load_vec<float, V>(a.conv + (long)j * a.width + c, w);
    #pragma unroll
    for (int i = 0; i < V; ++i) y[i] += w[i] * x[i];
    if (slot >= 0 && j > 0) store_vec<T, V>(tail + (long)(j - 1) * a.width, x);
  }
  if (slot >= 0 && past > 0)
    store_vec<T, V>(tail + (long)(past - 1) * a.width, h);
  store_vec<T, V>(out, y);
}

template <typename T, int V, bool ADD, typename Value>
DEV void between_sublayers(const Between<T>& a, long t, float* scratch,
                           Value value) {
  constexpr int HELD = 4;
  const int tid = threadIdx.x, n = a.width;
  float* res = a.residual + t * n;
  float held[HELD][V], ss = 0.f;
  auto squares = [&](const float* x) {
    #pragma unroll
    for (int j = 0; j < V; ++j) ss += x[j] * x[j];
  };
  // body(c, held or null) for the columns of this thread
  auto columns = [&](auto body) {
    #pragma unroll
    for (int i = 0; i < HELD; ++i) {
      const int c = (i * 256 + tid) * V;
      if (c < n) body(c, held[i], true);
    }
    for (int c = (HELD * 256 + tid) * V; c < n; c += 256 * V) {
      float x[V];
      body(c, x, false);
    }
  };
  if constexpr (ADD) {
    columns([&](int c, float* x, bool) {
      value(c, x);
      squares(x);
    });
    const float rs =
        1.f / sqrtf(block_reduce_sum_256(ss, scratch) / n + a.eps);
    ss = 0.f;
    columns([&](int c, float* x, bool is_held) {
      float w[V], r[V];
      if (!is_held) value(c, x);
      load_vec<float, V>(a.post + c, w);
      load_vec<float, V>(res + c, r);
      #pragma unroll
      for (int j = 0; j < V; ++j) x[j] = r[j] + x[j] * rs * w[j];
      store_vec<float, V>(res + c, x);
      squares(x);
    });
  } else {
    columns([&](int c, float* x, bool) {
      load_vec<float, V>(res + c, x);
      squares(x);
    });
  }
  const float rs = 1.f / sqrtf(block_reduce_sum_256(ss, scratch) / n + a.eps);
  columns([&](int c, float* x, bool is_held) {
    float w[V];
    if (!is_held) load_vec<float, V>(res + c, x);
    load_vec<float, V>(a.pre + c, w);
    #pragma unroll
    for (int j = 0; j < V; ++j) x[j] *= rs * w[j];
    store_input<T, V>(a, t, c, x);
  });
}
