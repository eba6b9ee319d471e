// Activations of a product's rows, which may be columns of wider ones, CDNA4 (gfx950):
//  * silu_glu: [gate | up] -> silu(gate) up
//  * relu2: max(x, 0)^2
// One pass, 16-byte accesses when widths and places allow; arithmetic in fp32, storage bf16 or fp32.
#include "ds_hip.h"

namespace {

enum : int { SILU_GLU = 1, RELU2 = 2 };

__device__ __forceinline__ float silu_glu_f(float g, float u) { return g / (1.f + expf(-g)) * u; }
__device__ __forceinline__ float relu2_f(float x) {
  x = fmaxf(x, 0.f);
  return x * x;
}

template <typename T, int ACT, bool VEC>
__global__ void __launch_bounds__(256) row_act_kernel(const T* __restrict__ x, int64_t ld, T* __restrict__ out, int64_t rows,
                                                      int F) {
  const int per = VEC ? F / 8 : F;
  const int64_t total = rows * per;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
    const int64_t r = i / per;
    const int c = (int)(i - r * per) * (VEC ? 8 : 1);
    const T* p = x + r * ld + c;
    if constexpr (VEC) {
      float a[8], b[8];
      Vec8<T>::load(p, a);
      if constexpr (ACT == SILU_GLU) Vec8<T>::load(p + F, b);
#pragma unroll
      for (int j = 0; j < 8; ++j) a[j] = ACT == SILU_GLU ? silu_glu_f(a[j], b[j]) : relu2_f(a[j]);
      Vec8<T>::store(out + r * F + c, a);
    } else {
      out[r * F + c] = (T)(ACT == SILU_GLU ? silu_glu_f((float)p[0], (float)p[F]) : relu2_f((float)p[0]));
    }
  }
}

template <typename T, int ACT>
int launch(const void* x, int64_t ld, void* out, int64_t rows, int F, hipStream_t st) {
  const bool vec = F % 8 == 0 && ld % 8 == 0 && ((uintptr_t)x & 15) == 0;
  const int grid = ds_grid_for(rows * (vec ? F / 8 : F), 256, 256 * 16);
  if (vec)
    hipLaunchKernelGGL((row_act_kernel<T, ACT, true>), dim3(grid), dim3(256), 0, st, (const T*)x, ld, (T*)out, rows, F);
  else
    hipLaunchKernelGGL((row_act_kernel<T, ACT, false>), dim3(grid), dim3(256), 0, st, (const T*)x, ld, (T*)out, rows, F);
  DS_CHECK_LAUNCH();
  return 0;
}

}  // namespace

// x: rows ld elements apart, of F columns (gated: 2 F) -> out [rows, F]
extern "C" int ds_row_act(const void* x, int64_t ld, void* out, int64_t rows, int F, int act, int dtype, hipStream_t st) {
  if (rows <= 0) return 0;
  if (F <= 0 || ld < (act == SILU_GLU ? 2 : 1) * (int64_t)F) return (int)hipErrorInvalidValue;
#define GO(T)                                                               \
  {                                                                         \
    if (act == SILU_GLU) return launch<T, SILU_GLU>(x, ld, out, rows, F, st); \
    if (act == RELU2) return launch<T, RELU2>(x, ld, out, rows, F, st);     \
  }
  if (dtype == DS_F32) GO(float)
  if (dtype == DS_BF16) GO(bf16)
#undef GO
  return (int)hipErrorInvalidValue;
}
