// Host-side operand checks shared by the hybrid decoders' op registrations.
#pragma once

#include <torch/library.h>
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>
#include <c10/core/DeviceGuard.h>

#include <optional>

namespace {

using at::Tensor;
using OptT = std::optional<Tensor>;

[[maybe_unused]] hipStream_t cur() { return c10::hip::getCurrentHIPStream().stream(); }

// model dtype: bf16 or fp32, unit inner stride
[[maybe_unused]] bool model_f32(const Tensor& t, const char* n) {
  TORCH_CHECK(t.is_cuda(), n, " must be a GPU tensor");
  TORCH_CHECK(t.scalar_type() == at::kBFloat16 || t.scalar_type() == at::kFloat, n, " must be bf16 or fp32");
  TORCH_CHECK(t.dim() == 0 || t.stride(-1) == 1, n, " needs a unit inner stride");
  return t.scalar_type() == at::kFloat;
}
[[maybe_unused]] void like(const Tensor& t, const Tensor& ref, const char* n) {
  model_f32(t, n);
  TORCH_CHECK(t.scalar_type() == ref.scalar_type(), n, " has another dtype than its operands");
}
[[maybe_unused]] const float* f32_of(const Tensor& t, int64_t numel, const char* n) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kFloat && t.is_contiguous() && t.numel() == numel, n,
              " must be a contiguous fp32 GPU tensor of ", numel, " elements");
  return t.data_ptr<float>();
}
[[maybe_unused]] const int* i32_of(const Tensor& t, const char* n) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kInt && t.is_contiguous(), n, " must be contiguous int32 on the GPU");
  return t.data_ptr<int>();
}
// rows of 16-B aligned vectors (the kernels' widest loads)
[[maybe_unused]] void aligned16(const Tensor& t, const char* n) {
  TORCH_CHECK(reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0, n, " must be 16-B aligned");
}

}  // namespace
