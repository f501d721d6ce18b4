// What the binding files share: shape checks, typed pointers, dispatch on the
// activations' type.
#pragma once

#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>

#include "typed.h"

namespace {

using torch::Tensor;
using OptTensor = std::optional<Tensor>;

hipStream_t stream() { return at::cuda::getCurrentCUDAStream().stream(); }

template <class T> struct Scalar;
template <> struct Scalar<float> { static constexpr auto type = torch::kFloat32; };
template <> struct Scalar<bf16_t> { static constexpr auto type = torch::kBFloat16; };

void check(const Tensor& t, torch::ScalarType type, const char* name,
           bool contiguous = true) {
  TORCH_CHECK(t.is_cuda(), name, " must be on the GPU");
  TORCH_CHECK(t.scalar_type() == type, name, " must be ", type, ", is ",
              t.scalar_type());
  TORCH_CHECK(!contiguous || t.is_contiguous(), name, " must be contiguous");
}

template <class T>
T* ptr(const Tensor& t) { return reinterpret_cast<T*>(t.data_ptr()); }
template <class T>
T* ptr(const OptTensor& t) { return t ? ptr<T>(*t) : nullptr; }

// [rows, n] view whose rows are `stride(0)` apart
void check_rows(const Tensor& t, torch::ScalarType type, const char* name) {
  check(t, type, name, false);
  TORCH_CHECK(t.dim() == 2 && (t.stride(1) == 1 || t.size(1) == 1), name,
              " must be [rows, n] with contiguous rows");
}

void post(const char* op) {
  const hipError_t e = hipGetLastError();
  TORCH_CHECK(e == hipSuccess, op, ": launch failed: ", hipGetErrorString(e));
}

Glu glu_of(const std::string& name) {
  if (name == "relu") return Glu::RELU;
  if (name == "clamped") return Glu::CLAMPED;
  TORCH_CHECK(name == "silu", "unknown gated feed-forward ", name);
  return Glu::SILU;
}

template <class F>
void by_type(const Tensor& t, F f) {
  if (t.scalar_type() == torch::kBFloat16) f(bf16_t{});
  else if (t.scalar_type() == torch::kFloat32) f(float{});
  else TORCH_CHECK(false, "activations must be float32 or bfloat16");
}

}  // namespace

void bind_mixers(pybind11::module& m);       // bindings_mixers.hip
