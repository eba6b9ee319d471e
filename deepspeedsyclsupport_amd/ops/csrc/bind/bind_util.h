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
[[maybe_unused]] const float* opt_f32(const OptT& t, int64_t n, const char* name) { return has(t) ? f32(*t, n, name) : nullptr; }
[[maybe_unused]] const double* f64(const Tensor& t, const char* name) {
  need(t, name);
  TORCH_CHECK(t.scalar_type() == at::kDouble, name, ": fp64");
  return t.data_ptr<double>();
}
// A matrix whose rows may lie further apart than they are wide
[[maybe_unused]] void need_rows(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.dim() == 2 && t.stride(1) == 1 && (t.size(0) <= 1 || t.stride(0) >= t.size(1)), name,
              " must be a device matrix with contiguous rows");
}
}  // namespace
