// Shared parts of the binding files: argument checks, element type dispatch.
#pragma once

#include <torch/extension.h>

#include <c10/hip/HIPStream.h>
#include <hip/hip_bf16.h>

#include <stdexcept>
#include <type_traits>

#include "side.h"

using bf16 = __hip_bfloat16;

inline hipStream_t stream() {
  return c10::hip::getCurrentHIPStream().stream();
}

inline void check(const torch::Tensor& t, torch::ScalarType dt, const char* name) {
  TORCH_CHECK(t.is_cuda(), name, " must be on GPU");
  TORCH_CHECK(t.is_contiguous(), name, " must be contiguous");
  TORCH_CHECK(t.scalar_type() == dt, name, " has wrong dtype");
}

template <typename T> T* ptr(const torch::Tensor& t) {
  return reinterpret_cast<T*>(t.data_ptr());
}

// run f with a null pointer of the element type that t has
template <typename F> void by_dtype(const torch::Tensor& t, F f) {
  if (t.scalar_type() == torch::kBFloat16)
    f((bf16*)nullptr);
  else if (t.scalar_type() == torch::kFloat32)
    f((float*)nullptr);
  else
    TORCH_CHECK(false, "element type must be bfloat16 or float32");
}

#define ELEM(tag) std::remove_pointer_t<decltype(tag)>

// [T, n] view with unit column stride of one projection buffer
inline void check_rows(const torch::Tensor& t, torch::ScalarType dt, long rows,
                long cols, long stride, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == dt && t.dim() == 2 &&
                  t.size(0) == rows && t.size(1) == cols &&
                  t.stride(1) == 1 && t.stride(0) == stride,
              name, " must be a [", rows, ", ", cols,
              "] view of the projection buffer");
}

inline void check_param(const torch::Tensor& t, long numel, const char* name) {
  check(t, torch::kFloat32, name);
  TORCH_CHECK(t.numel() == numel, name, " must have ", numel, " elements");
}

// tiles [num_tiles, 2] of portions listed by seq_start; one table row each
inline void check_tiles(const torch::Tensor& tiles, const torch::Tensor& seq_start,
                 long seqs) {
  check(tiles, torch::kInt32, "tiles");
  check(seq_start, torch::kInt32, "seq_start");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 2, "tiles");
  TORCH_CHECK(seq_start.numel() == seqs + 1, "seq_start");
}

inline float* opt(const c10::optional<torch::Tensor>& t) {
  return t.has_value() ? ptr<float>(*t) : nullptr;
}

// side activation: x and out [rows, n] column views, or neither
template <typename T>
SideRelu<T> side_of(const c10::optional<torch::Tensor>& x,
                    const c10::optional<torch::Tensor>& out, long rows,
                    torch::ScalarType dt) {
  TORCH_CHECK(x.has_value() == out.has_value(), "side activation");
  if (!x.has_value()) return {};
  const long n = x->size(1);
  check_rows(*x, dt, rows, n, x->stride(0), "side x");
  check_rows(*out, dt, rows, n, out->stride(0), "side out");
  return make_side<T>(ptr<T>(*x), ptr<T>(*out), x->stride(0), out->stride(0),
                      (int)n);
}
