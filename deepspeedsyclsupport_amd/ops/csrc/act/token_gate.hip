// Elementwise steps of decoders with a token-side input, CDNA4 (gfx950):
//  * gelu: the exact (error function) gelu of an ungated feed-forward;
//  * token_gate: gelu_tanh(g) * e, with e a slice of the token's row in a side embedding.
// 16-byte accesses when the width allows; arithmetic in fp32, storage bf16 or fp32.
#include "ds_hip.h"

namespace {

__device__ __forceinline__ float gelu_erf_f(float x) { return 0.5f * x * (1.f + erff(x * 0.70710678118654752f)); }
__device__ __forceinline__ float gelu_tanh_f(float x) {
  return 0.5f * x * (1.f + tanhf(0.79788456080286536f * fmaf(0.044715f * x * x, x, x)));
}

template <typename T>
__global__ void __launch_bounds__(256) gelu_kernel(const T* __restrict__ x, T* __restrict__ out, int64_t n) {
  const int64_t vec = n / 8;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < vec; i += (int64_t)gridDim.x * 256) {
    float v[8];
    Vec8<T>::load(x + i * 8, v);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = gelu_erf_f(v[j]);
    Vec8<T>::store(out + i * 8, v);
  }
  if (blockIdx.x == 0)
    for (int64_t i = vec * 8 + threadIdx.x; i < n; i += 256) out[i] = (T)gelu_erf_f((float)x[i]);
}

template <typename T>
__global__ void __launch_bounds__(256) token_gate_kernel(const T* __restrict__ g, const int* __restrict__ ids,
                                                         const T* __restrict__ table, int64_t stride, T* __restrict__ out,
                                                         int64_t n, int D) {
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) {
    const int64_t t = i / D;
    out[i] = (T)(gelu_tanh_f((float)g[i]) * (float)table[ids[t] * stride + (i - t * D)]);
  }
}

}  // namespace

extern "C" int ds_gelu(const void* x, void* out, int64_t n, int dtype, hipStream_t st) {
  if (n <= 0) return 0;
  const int grid = ds_grid_for((n + 7) / 8, 256, 256 * 16);
  if (dtype == DS_F32)
    hipLaunchKernelGGL((gelu_kernel<float>), dim3(grid), dim3(256), 0, st, (const float*)x, (float*)out, n);
  else if (dtype == DS_BF16)
    hipLaunchKernelGGL((gelu_kernel<bf16>), dim3(grid), dim3(256), 0, st, (const bf16*)x, (bf16*)out, n);
  else return (int)hipErrorInvalidValue;
  DS_CHECK_LAUNCH();
  return 0;
}

// g [tokens, D]; table: the slice's first column, rows `stride` apart
extern "C" int ds_token_gate(const void* g, const int* ids, const void* table, int64_t stride, void* out, int64_t tokens,
                             int D, int dtype, hipStream_t st) {
  const int64_t n = tokens * D;
  if (n <= 0) return 0;
  const int grid = ds_grid_for(n, 256, 256 * 16);
  if (dtype == DS_F32)
    hipLaunchKernelGGL((token_gate_kernel<float>), dim3(grid), dim3(256), 0, st, (const float*)g, ids, (const float*)table,
                       stride, (float*)out, n, D);
  else if (dtype == DS_BF16)
    hipLaunchKernelGGL((token_gate_kernel<bf16>), dim3(grid), dim3(256), 0, st, (const bf16*)g, ids, (const bf16*)table,
                       stride, (bf16*)out, n, D);
  else return (int)hipErrorInvalidValue;
  DS_CHECK_LAUNCH();
  return 0;
}
