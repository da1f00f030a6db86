// Common helpers for the gfx950 (CDNA4, MI355X) kernels.
//
// These kernels are written natively for CDNA4 — wave64, 4 SIMD-32/CU,
// 160 KiB LDS, HBM3E — per /opt/skills/guides/cdna_hip_programming.md.
// No CUDA compatibility layer, no hipify, gfx950 only.
#pragma once

#include <hip/hip_runtime.h>
#include <hip/hip_bf16.h>

#define WAVE 64
#define DEV __device__ __forceinline__

using bf16 = __hip_bfloat16;

// ---- bf16 <-> f32 bit tricks (one ushort per value) --------------------
DEV float bf2f(unsigned short u) {
  union { unsigned int i; float f; } c;
  c.i = (unsigned int)u << 16;
  return c.f;
}

DEV unsigned short f2bf(float f) {
  union { float f; unsigned int i; } c;
  c.f = f;
  // round-to-nearest-even
  unsigned int lsb = (c.i >> 16) & 1;
  c.i += 0x7fffu + lsb;
  return (unsigned short)(c.i >> 16);
}

// 8 bf16 loaded as one 16-byte vector (guideline 13: always vectorize bf16)
struct bf16x8 { uint4 raw; };

DEV bf16x8 load_bf16x8(const bf16* p) {
  bf16x8 r;
  r.raw = *reinterpret_cast<const uint4*>(p);
  return r;
}

DEV void store_bf16x8(bf16* p, const bf16x8& v) {
  *reinterpret_cast<uint4*>(p) = v.raw;
}

DEV float bf16x8_get(const bf16x8& v, int i) {
  unsigned int w = (&v.raw.x)[i >> 1];
  return bf2f((unsigned short)(i & 1 ? w >> 16 : w & 0xffff));
}

DEV void bf16x8_set(bf16x8& v, int i, float f) {
  unsigned int* w = &(&v.raw.x)[i >> 1];
  unsigned short b = f2bf(f);
  if (i & 1) *w = (*w & 0x0000ffffu) | ((unsigned int)b << 16);
  else       *w = (*w & 0xffff0000u) | b;
}

// ---- element type access: kernels templated on bf16 | float -------------
template <typename T> struct Elem;

template <> struct Elem<bf16> {
  static DEV float ld(const bf16* p) {
    return bf2f(*reinterpret_cast<const unsigned short*>(p));
  }
  static DEV void st(bf16* p, float f) {
    *reinterpret_cast<unsigned short*>(p) = f2bf(f);
  }
  static DEV float4 ld4(const bf16* p) {
    const ushort4 u = *reinterpret_cast<const ushort4*>(p);
    return make_float4(bf2f(u.x), bf2f(u.y), bf2f(u.z), bf2f(u.w));
  }
  static DEV void st4(bf16* p, float4 f) {
    *reinterpret_cast<ushort4*>(p) =
        make_ushort4(f2bf(f.x), f2bf(f.y), f2bf(f.z), f2bf(f.w));
  }
};

template <> struct Elem<float> {
  static DEV float ld(const float* p) { return *p; }
  static DEV void st(float* p, float f) { *p = f; }
  static DEV float4 ld4(const float* p) {
    return *reinterpret_cast<const float4*>(p);
  }
  static DEV void st4(float* p, float4 f) {
    *reinterpret_cast<float4*>(p) = f;
  }
};

// V consecutive elements (V = 1, 4 or 8, which need alignment to V elements)
template <typename T, int V> DEV void load_vec(const T* p, float* f) {
  if constexpr (V == 8) {
    load_vec<T, 4>(p, f);
    load_vec<T, 4>(p + 4, f + 4);
  } else if constexpr (V == 4) {
    const float4 v = Elem<T>::ld4(p);
    f[0] = v.x; f[1] = v.y; f[2] = v.z; f[3] = v.w;
  } else {
    f[0] = Elem<T>::ld(p);
  }
}
template <typename T, int V> DEV void store_vec(T* p, const float* f) {
  if constexpr (V == 8) {
    store_vec<T, 4>(p, f);
    store_vec<T, 4>(p + 4, f + 4);
  } else if constexpr (V == 4)
    Elem<T>::st4(p, make_float4(f[0], f[1], f[2], f[3]));
  else
    Elem<T>::st(p, f[0]);
}

// Transcendentals: the bf16 kernels take the hardware exponential (absolute
// error ~1e-7, far below a bf16 step), the float kernels the library ones.
template <typename T> struct Fn;
template <> struct Fn<bf16> {
  static DEV float exp(float x) { return __expf(x); }
  static DEV float tanh(float x) {
    return 1.f - 2.f / (1.f + __expf(2.f * x));
  }
};
template <> struct Fn<float> {
  static DEV float exp(float x) { return expf(x); }
  static DEV float tanh(float x) { return tanhf(x); }
};

// clamped gated unit: g sigmoid(1.702 g) (u + 1) with g = min(gate, limit) and
// u clamped to +-limit
template <typename T> DEV float clamped_unit(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.f + Fn<T>::exp(-1.702f * g)) * (u + 1.f);
}

// log(sigmoid(z)) without overflow for either sign of z
DEV float log_sigmoid(float z) {
  return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}

// ---- matrix-core operands ----------------------------------------------
typedef __attribute__((ext_vector_type(8))) short short8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;
typedef __attribute__((ext_vector_type(16))) float f32x16_t;

// two floats -> packed bf16 (round to nearest even), one v_cvt_pk_bf16_f32.
// Not as inline assembly: the compiler would not see that its operands may
// come straight from a transcendental or matrix instruction, whose results
// need a wait before they are read.
DEV unsigned cvt_pk_bf16(float a, float b) {
  typedef __attribute__((ext_vector_type(2))) float float2_t;
  typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2_t;
  union { bf16x2_t v; unsigned u; } r;
  r.v = __builtin_convertvector(float2_t{a, b}, bf16x2_t);
  return r.u;
}

// f = hi + lo to ~16 bits of mantissa: a float operand as two bf16 ones
DEV void split_bf16x8(const float* f, short8_t* hi, short8_t* lo) {
  union { unsigned u[4]; short8_t v; } h, l;
  #pragma unroll
  for (int i = 0; i < 4; ++i) {
    h.u[i] = cvt_pk_bf16(f[2 * i], f[2 * i + 1]);
    l.u[i] = cvt_pk_bf16(f[2 * i] - bf2f((unsigned short)(h.u[i] & 0xffff)),
                         f[2 * i + 1] - bf2f((unsigned short)(h.u[i] >> 16)));
  }
  *hi = h.v;
  *lo = l.v;
}

DEV float bf16x8_at(const short8_t& v, int i) {
  return bf2f((unsigned short)v[i]);
}

DEV f32x4_t mfma16(short8_t a, short8_t b, f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
DEV f32x16_t mfma32(short8_t a, short8_t b, f32x16_t c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0);
}

// ---- reductions ---------------------------------------------------------
DEV float wave_reduce_sum(float v) {
  #pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o);
  return v;
}

DEV float wave_reduce_max(float v) {
  #pragma unroll
  for (int o = 32; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o));
  return v;
}

// 256-thread block reduce; scratch must hold >= 4 floats; result valid in
// every thread.  Caller owns barrier hygiene around reuse of scratch.
DEV float block_reduce_sum_256(float v, float* scratch) {
  v = wave_reduce_sum(v);
  const int wid = threadIdx.x >> 6;
  if ((threadIdx.x & 63) == 0) scratch[wid] = v;
  __syncthreads();
  float total = scratch[0] + scratch[1] + scratch[2] + scratch[3];
  __syncthreads();
  return total;
}

DEV float block_reduce_max_256(float v, float* scratch) {
  v = wave_reduce_max(v);
  const int wid = threadIdx.x >> 6;
  if ((threadIdx.x & 63) == 0) scratch[wid] = v;
  __syncthreads();
  float total = fmaxf(fmaxf(scratch[0], scratch[1]),
                      fmaxf(scratch[2], scratch[3]));
  __syncthreads();
  return total;
}

#define HIP_CHECK(expr)                                                     \
  do {                                                                      \
    hipError_t _e = (expr);                                                 \
    if (_e != hipSuccess)                                                   \
      throw std::runtime_error(std::string("HIP error: ") +                 \
                               hipGetErrorString(_e));                      \
  } while (0)
