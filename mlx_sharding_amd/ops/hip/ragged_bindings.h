// What the files with Python bindings of the ragged-batch kernels share: checks
// of device, type, shape and alignment, made before anything is launched.
#pragma once

#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

#include "ragged_common.h"

namespace {

using torch::Tensor;

[[maybe_unused]] hipStream_t stream() { return c10::hip::getCurrentHIPStream().stream(); }

[[maybe_unused]] bool is_f32(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda(), name, " must be on the GPU");
  TORCH_CHECK(t.scalar_type() == torch::kFloat32 ||
                  t.scalar_type() == torch::kBFloat16,
              name, " must be float32 or bfloat16");
  return t.scalar_type() == torch::kFloat32;
}

[[maybe_unused]] void check_like(const Tensor& t, const Tensor& as, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == as.scalar_type(), name,
              " must be on the GPU with the activations' type");
}

[[maybe_unused]] void check_f32(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kFloat32 &&
                  t.is_contiguous(),
              name, " must be contiguous float32 on the GPU");
}

[[maybe_unused]] const int* ints(const Tensor& t, int64_t at_least, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kInt32 &&
                  t.is_contiguous() && t.numel() >= at_least,
              name, " must be contiguous int32 on the GPU with at least ",
              at_least, " elements");
  return t.data_ptr<int>();
}

// [N, C] with unit column stride; returns the row stride
[[maybe_unused]] long rows2(const Tensor& t, const char* name) {
  TORCH_CHECK(t.dim() == 2 && (t.stride(1) == 1 || t.size(1) == 1), name,
              " must be [rows, columns] with unit column stride");
  return t.size(0) > 1 ? t.stride(0) : std::max<long>(t.stride(0), t.size(1));
}

[[maybe_unused]] void aligned16(const Tensor& t, const char* name) {
  TORCH_CHECK(((uintptr_t)t.data_ptr()) % 16 == 0, name,
              " must be 16-byte aligned");
}

[[maybe_unused]] bool whole8(const Tensor& t, long stride) {
  return ((uintptr_t)t.data_ptr()) % 16 == 0 && stride % 8 == 0;
}

}  // namespace

void bind_recurrent(pybind11::module_& m);
void bind_experts(pybind11::module_& m);
