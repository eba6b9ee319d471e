// A recurrent mixer's read-out with its output gate, CDNA4 (gfx950). The read-out's equal parts are divided by their own root
// mean squares, times an optional weight, with the gate's activation multiplied in before or after:
//     GATE_SILU_BEFORE     y silu(gate), then the norm
//     GATE_SIGMOID_AFTER   the norm, then sigmoid(gate)
//     GATE_SILU_AFTER      the norm, then silu(gate)
// The result may be some columns of a wider row (read-outs of several mixers side by side).
//
// HBM-bound: every operand is read once with 16-byte accesses and kept in registers; parts of up to 256 columns share a wave.
// Rows no vector width divides take a plain version that reads y again.
#include "ds_hip.h"

namespace {

enum : int { GATE_SIGMOID_AFTER = 0, GATE_SILU_BEFORE = 1, GATE_SILU_AFTER = 2 };

__device__ __forceinline__ float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }

// NT threads per (token, part) of P columns, E x 8 elements per thread; PB such groups per workgroup (NT up to 64)
template <typename T, int NT, int E>
__global__ void __launch_bounds__(NT < 256 ? 256 : NT) gated_norm_kernel(const T* __restrict__ y, const T* __restrict__ gate,
                                                                         int64_t gstride, const float* __restrict__ w,
                                                                         T* __restrict__ out, int64_t ostride, int64_t items,
                                                                         int C, int P, int parts, float eps, int mode) {
  constexpr int PB = NT < 256 ? 256 / NT : 1;
  __shared__ float red[PB > 1 ? 1 : NT / 64];
  const int64_t item = (int64_t)blockIdx.x * PB + threadIdx.x / NT;
  if (PB > 1 && item >= items) return;  // whole groups: they only exchange values among themselves
  const bool before = mode == GATE_SILU_BEFORE, sig = mode == GATE_SIGMOID_AFTER;
  const int tid = threadIdx.x % NT;
  const int64_t t = item / parts;
  const int c0 = (int)(item % parts) * P;
  float v[E][8], g[E][8], ss = 0.f;
#pragma unroll
  for (int i = 0; i < E; ++i) {
    const int c = (tid + i * NT) * 8, cc = c0 + (c < P ? c : 0);
    Vec8<T>::load(y + t * C + cc, v[i]);
    Vec8<T>::load(gate + t * gstride + cc, g[i]);
  }
#pragma unroll
  for (int i = 0; i < E; ++i) {
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      g[i][j] = (sig ? 1.f : g[i][j]) * sigmoid_f(g[i][j]);
      if (before) v[i][j] *= g[i][j];
    }
    if ((tid + i * NT) * 8 < P) {
#pragma unroll
      for (int j = 0; j < 8; ++j) ss = fmaf(v[i][j], v[i][j], ss);
    }
  }
  if constexpr (PB > 1) {
#pragma unroll
    for (int o = NT / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
  } else {
    ss = block_sum(ss, red);
  }
  const float rs = 1.f / sqrtf(ss / (float)P + eps);
#pragma unroll
  for (int i = 0; i < E; ++i) {
    const int c = (tid + i * NT) * 8;
    if (c >= P) continue;
    float ww[8] = {1.f, 1.f, 1.f, 1.f, 1.f, 1.f, 1.f, 1.f};
    if (w) Vec8<float>::load(w + c0 + c, ww);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[i][j] *= rs * ww[j] * (before ? 1.f : g[i][j]);
    Vec8<T>::store(out + t * ostride + c0 + c, v[i]);
  }
}

template <typename T>
__global__ void __launch_bounds__(256) gated_norm_any_kernel(const T* __restrict__ y, const T* __restrict__ gate,
                                                             int64_t gstride, const float* __restrict__ w,
                                                             T* __restrict__ out, int64_t ostride, int C, int P,
                                                             int parts, float eps, int mode) {
  __shared__ float red[4];
  const bool before = mode == GATE_SILU_BEFORE;
  const int64_t t = blockIdx.x / parts;
  const int c0 = (int)(blockIdx.x % parts) * P;
  const T* yr = y + t * C + c0;
  const T* gr = gate + t * gstride + c0;
  float ss = 0.f;
  for (int c = threadIdx.x; c < P; c += 256) {
    const float g = (float)gr[c], v = (float)yr[c] * (before ? g * sigmoid_f(g) : 1.f);
    ss = fmaf(v, v, ss);
  }
  const float rs = 1.f / sqrtf(block_sum(ss, red) / (float)P + eps);
  for (int c = threadIdx.x; c < P; c += 256) {
    const float g = (float)gr[c], s = sigmoid_f(g);
    out[t * ostride + c0 + c] = (T)((float)yr[c] * rs * (w ? w[c0 + c] : 1.f) * (mode == GATE_SIGMOID_AFTER ? s : g * s));
  }
}

template <typename T>
int gated_norm(const void* y, const void* gate, int64_t gstride, const float* w, void* out, int64_t ostride,
               int64_t tokens, int C, int parts, float eps, int mode, hipStream_t st) {
  const int P = C / parts;
  const int64_t items = tokens * parts;
  const bool vec = P % 8 == 0 && gstride % 8 == 0 && ((uintptr_t)gate & 15) == 0 && ostride % 8 == 0 &&
                   ((uintptr_t)out & 15) == 0 && P <= 32768;
#define GO(NT, E)                                                                                                     \
  hipLaunchKernelGGL((gated_norm_kernel<T, NT, E>), dim3((unsigned)((items * NT + (NT < 256 ? 255 : NT - 1)) /           \
                     (NT < 256 ? 256 : NT))), dim3(NT < 256 ? 256 : NT), 0, st, (const T*)y, (const T*)gate, gstride, w,   \
                     (T*)out, ostride, items, C, P, parts, eps, mode)
  if (!vec)
    hipLaunchKernelGGL((gated_norm_any_kernel<T>), dim3((unsigned)items), dim3(256), 0, st, (const T*)y, (const T*)gate,
                       gstride, w, (T*)out, ostride, C, P, parts, eps, mode);
  else if (P <= 64) GO(8, 1);
  else if (P <= 128) GO(16, 1);
  else if (P <= 256) GO(32, 1);
  else if (P <= 512) GO(64, 1);
  else if (P <= 1024) GO(64, 2);
  else if (P <= 2048) GO(256, 1);
  else if (P <= 4096) GO(256, 2);
  else if (P <= 8192) GO(512, 2);
  else if (P <= 16384) GO(1024, 2);
  else GO(1024, 4);
#undef GO
  DS_CHECK_LAUNCH();
  return 0;
}

}  // namespace

// gate, out: row t starts at gate + t * gstride, out + t * ostride; w null: no weight
extern "C" int ds_gated_norm(const void* y, const void* gate, int64_t gstride, const float* w, void* out, int64_t ostride,
                             int64_t tokens, int C, int parts, float eps, int mode, int dtype, hipStream_t st) {
  if (tokens <= 0) return 0;
  if (C <= 0 || parts <= 0 || C % parts || ostride < C || mode < 0 || mode > 2 || tokens * parts > INT32_MAX) return (int)hipErrorInvalidValue;
  if (dtype == DS_F32) return gated_norm<float>(y, gate, gstride, w, out, ostride, tokens, C, parts, eps, mode, st);
  if (dtype == DS_BF16) return gated_norm<bf16>(y, gate, gstride, w, out, ostride, tokens, C, parts, eps, mode, st);
  return (int)hipErrorInvalidValue;
}
