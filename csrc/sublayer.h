// Between two sublayers, one row by a workgroup:
//
//   residual += rms(y) * post          (not before the first sublayer), or
//   residual += y                      (no norm after a sublayer)
//   h = rms(residual) * pre, rounded to T
//   out = h, or for a decoded token h + sum_j conv[j] * (input taps-1-j ago)
//
// y comes from value(c, y[V]), columns [c, c + V).  The residual and the norm
// and convolution weights are float.  The inputs that the convolution looks
// back at are kept in tail[slot], oldest first; those from before position 0
// count as zero whatever the slot holds.
//
// Without the convolution rows are many: 256 threads hold up to 4 * V columns
// each.  With it they are few and latency counts: as many threads as a row
// has column groups, and all that does not depend on the sums is loaded
// ahead.  Longer rows are read again.
#pragma once

#include <type_traits>

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

// RUN(V, threads, with convolution) for a Between named a
#define BY_WIDTH(RUN)                                                       \
  if (!a.conv) {                                                            \
    if (a.width % 4 == 0) { RUN(4, 256, false); }                           \
    else { RUN(1, 256, false); }                                            \
  } else if (a.width % 4) { RUN(1, 1024, true); }                           \
  else if (a.width <= 1024) { RUN(4, 256, true); }                          \
  else if (a.width <= 2048) { RUN(4, 512, true); }                          \
  else { RUN(4, 1024, true); }

// f as it reads back after a store to T
template <typename T> DEV float as_elem(float f) {
  if constexpr (sizeof(T) == 2) return bf2f(f2bf(f));
  else return f;
}

template <int NT> DEV float sum_over(float v) {
  __shared__ float part[NT / 64];
  v = wave_reduce_sum(v);
  if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = v;
  __syncthreads();
  v = 0.f;
  #pragma unroll
  for (int i = 0; i < NT / 64; ++i) v += part[i];
  __syncthreads();
  return v;
}

// the convolution of one column group: weights and past inputs of up to
// AHEAD taps are loaded by the constructor
template <typename T, int V> struct TokenConv {
  static constexpr int AHEAD = 4;
  const Between<T>& a;
  int past, slot;
  long first;               // position of the oldest past input
  float w[AHEAD][V], x[AHEAD - 1][V];

  DEV TokenConv(const Between<T>& a, long t, int c) : a(a) {
    past = a.taps - 1;
    slot = a.slots[t];
    first = a.positions[t] - past;
    if (past >= AHEAD || c >= a.width) return;
    #pragma unroll
    for (int j = 0; j < AHEAD; ++j)
      if (j <= past) load_vec<float, V>(a.conv + (long)j * a.width + c, w[j]);
    #pragma unroll
    for (int j = 0; j < AHEAD - 1; ++j)
      if (j < past) load_past(j, c, x[j]);
  }
  DEV T* tail(int j, int c) const {
    return a.tail + ((long)slot * past + j) * a.width + c;
  }
  DEV void load_past(int j, int c, float* f) const {
    #pragma unroll
    for (int i = 0; i < V; ++i) f[i] = 0.f;
    if (slot >= 0 && first + j >= 0) load_vec<T, V>(tail(j, c), f);
  }
  // y += wj * past input j, which moves one place on
  DEV void tap(int j, int c, const float* wj, const float* f, float* y) const {
    #pragma unroll
    for (int i = 0; i < V; ++i) y[i] += wj[i] * f[i];
    if (slot >= 0 && j > 0) store_vec<T, V>(tail(j - 1, c), f);
  }
  // h becomes the output; `held` tells that column group c was loaded ahead
  DEV void apply(int c, float* h, bool held) const {
    float y[V];
    #pragma unroll
    for (int i = 0; i < V; ++i) y[i] = h[i] = as_elem<T>(h[i]);
    if (held && past < AHEAD) {
      #pragma unroll
      for (int j = 0; j < AHEAD - 1; ++j)
        if (j < past) tap(j, c, w[j], x[j], y);
      #pragma unroll
      for (int j = 0; j < AHEAD; ++j)
        if (j == past)
          #pragma unroll
          for (int i = 0; i < V; ++i) y[i] += w[j][i] * h[i];
    } else {
      float wj[V], f[V];
      for (int j = 0; j < past; ++j) {
        load_vec<float, V>(a.conv + (long)j * a.width + c, wj);
        load_past(j, c, f);
        tap(j, c, wj, f, y);
      }
      load_vec<float, V>(a.conv + (long)past * a.width + c, wj);
      #pragma unroll
      for (int i = 0; i < V; ++i) y[i] += wj[i] * h[i];
    }
    if (slot >= 0 && past > 0) store_vec<T, V>(tail(past - 1, c), h);
    #pragma unroll
    for (int i = 0; i < V; ++i) h[i] = y[i];
  }
};

template <typename T, int V> struct NoConv {
  DEV NoConv(const Between<T>&, long, int) {}
  DEV void apply(int, float*, bool) const {}
};

// how y enters the residual
enum { ADD_NOTHING, ADD_NORMED, ADD_PLAIN };

template <typename T, int V, int NT, bool CONV, int ADD, typename Value>
DEV void between_sublayers(const Between<T>& a, long t, Value value) {
  constexpr int HELD = CONV ? 1 : 4;
  const int tid = threadIdx.x, n = a.width;
  float* res = a.residual + t * n;
  float held[HELD][V], ss = 0.f;
  // loaded ahead of the sums for the first column group
  float pre0[V], post0[V], res0[V];
  const std::conditional_t<CONV, TokenConv<T, V>, NoConv<T, V>> conv(
      a, t, tid * V);
  if (CONV && tid * V < n) {
    load_vec<float, V>(a.pre + tid * V, pre0);
    if (ADD == ADD_NORMED) load_vec<float, V>(a.post + tid * V, post0);
    load_vec<float, V>(res + tid * V, res0);
  }
  auto squares = [&](const float* x) {
    #pragma unroll
    for (int j = 0; j < V; ++j) ss += x[j] * x[j];
  };
  auto fetch = [&](const float* p, const float* ahead, int c, bool is_held,
                   float* f) {
    if (CONV && is_held) {
      #pragma unroll
      for (int j = 0; j < V; ++j) f[j] = ahead[j];
    } else {
      load_vec<float, V>(p + c, f);
    }
  };
  // body(c, columns, held in registers) for the columns of this thread
  auto columns = [&](auto body) {
    #pragma unroll
    for (int i = 0; i < HELD; ++i) {
      const int c = (i * NT + tid) * V;
      if (c < n) body(c, held[i], true);
    }
    for (int c = (HELD * NT + tid) * V; c < n; c += NT * V) {
      float x[V];
      body(c, x, false);
    }
  };
  if constexpr (ADD == ADD_NORMED) {
    columns([&](int c, float* x, bool) {
      value(c, x);
      squares(x);
    });
    const float rs = 1.f / sqrtf(sum_over<NT>(ss) / n + a.eps);
    ss = 0.f;
    columns([&](int c, float* x, bool is_held) {
      float w[V], r[V];
      if (!is_held) value(c, x);
      fetch(a.post, post0, c, is_held, w);
      fetch(res, res0, c, is_held, r);
      #pragma unroll
      for (int j = 0; j < V; ++j) x[j] = r[j] + x[j] * rs * w[j];
      store_vec<float, V>(res + c, x);
      squares(x);
    });
  } else {
    columns([&](int c, float* x, bool is_held) {
      fetch(res, res0, c, is_held, x);
      if constexpr (ADD == ADD_PLAIN) {
        float y[V];
        value(c, y);
        #pragma unroll
        for (int j = 0; j < V; ++j) x[j] += y[j];
        store_vec<float, V>(res + c, x);
      }
      squares(x);
    });
  }
  const float rs = 1.f / sqrtf(sum_over<NT>(ss) / n + a.eps);
  columns([&](int c, float* x, bool is_held) {
    float w[V];
    if (!is_held) load_vec<float, V>(res + c, x);
    fetch(a.pre, pre0, c, is_held, w);
    #pragma unroll
    for (int j = 0; j < V; ++j) x[j] *= rs * w[j];
    conv.apply(c, x, is_held);
    store_vec<T, V>(a.out + t * n + c, x);
  });
}
