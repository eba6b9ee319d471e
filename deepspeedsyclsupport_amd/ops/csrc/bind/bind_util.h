// Argument checks shared by the small extension modules.
#pragma once
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>
#include <hip/hip_runtime_api.h>

#include <optional>

using torch::Tensor;
using OptT = std::optional<Tensor>;

namespace {
hipStream_t stream() { return at::hip::getCurrentHIPStream().stream(); }
void check(int rc, const char* what) { TORCH_CHECK(rc == 0, what, " failed: ", hipGetErrorString((hipError_t)rc)); }
int dcode(const Tensor& t) {
  if (t.scalar_type() == at::kFloat) return 0;
  TORCH_CHECK(t.scalar_type() == at::kBFloat16, "fp32 or bf16 tensors");
  return 1;
}
void need(const Tensor& t, const char* n) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous(), n, " must be a contiguous device tensor");
}
const float* f32(const Tensor& t, int64_t n, const char* name) {
  need(t, name);
  TORCH_CHECK(t.scalar_type() == at::kFloat && t.numel() == n, name, ": fp32 with ", n, " elements");
  return t.data_ptr<float>();
}
const int* i32(const Tensor& t, int64_t n, const char* name) {
  need(t, name);
  TORCH_CHECK(t.scalar_type() == at::kInt && t.numel() == n, name, ": int32 with ", n, " elements");
  return t.data_ptr<int>();
}
bool has(const OptT& t) { return t.has_value() && t->defined(); }
}  // namespace
