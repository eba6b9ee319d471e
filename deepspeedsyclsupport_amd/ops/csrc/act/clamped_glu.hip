// Clamped gated activation of a fused [gate | up] projection, CDNA4 (gfx950):
//   g = min(gate, limit), u = clamp(up, -limit, limit);   out = g * sigmoid(alpha * g) * (u + shift)
// One pass, 16-byte accesses when the width allows; arithmetic in fp32, storage bf16 or fp32.
#include "ds_hip.h"

namespace {

template <typename T, bool VEC>
__global__ void __launch_bounds__(256) clamped_glu_kernel(const T* __restrict__ gu, T* __restrict__ out, int64_t rows,
                                                          int F, float limit, float alpha, float shift) {
  const int per = VEC ? F / 8 : F;
  const int64_t total = rows * per;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
    const int64_t r = i / per;
    const int c = (int)(i - r * per) * (VEC ? 8 : 1);
    const T* g = gu + r * 2 * F + c;
    if constexpr (VEC) {
      float a[8], b[8];
      Vec8<T>::load(g, a);
      Vec8<T>::load(g + F, b);
#pragma unroll
      for (int j = 0; j < 8; ++j) a[j] = clamped_glu_f(a[j], b[j], limit, alpha, shift);
      Vec8<T>::store(out + r * F + c, a);
    } else {
      out[r * F + c] = (T)clamped_glu_f((float)g[0], (float)g[F], limit, alpha, shift);
    }
  }
}

template <typename T>
int launch(const void* gu, void* out, int64_t rows, int F, float limit, float alpha, float shift, hipStream_t st) {
  const bool vec = F % 8 == 0;
  const int grid = ds_grid_for(rows * (vec ? F / 8 : F), 256, 256 * 16);
  if (vec)
    hipLaunchKernelGGL((clamped_glu_kernel<T, true>), dim3(grid), dim3(256), 0, st, (const T*)gu, (T*)out, rows, F,
                       limit, alpha, shift);
  else
    hipLaunchKernelGGL((clamped_glu_kernel<T, false>), dim3(grid), dim3(256), 0, st, (const T*)gu, (T*)out, rows, F,
                       limit, alpha, shift);
  DS_CHECK_LAUNCH();
  return 0;
}

}  // namespace

extern "C" int ds_clamped_glu(const void* gu, void* out, int64_t rows, int F, float limit, float alpha, float shift,
                              int dtype, hipStream_t st) {
  if (rows <= 0) return 0;
  if (F <= 0) return (int)hipErrorInvalidValue;
  if (dtype == DS_F32) return launch<float>(gu, out, rows, F, limit, alpha, shift, st);
  if (dtype == DS_BF16) return launch<bf16>(gu, out, rows, F, limit, alpha, shift, st);
  return (int)hipErrorInvalidValue;
}
