// Residual of decoders that normalise sublayer outputs, CDNA4 (gfx950).
//
// One launch per sublayer boundary: x <- x + y / rms(y) * w on the fp32 residual, and x again in the storage type as the next
// sublayer's input; or, at the start of the model, x <- the token's embedding row. With a row list (the rows whose logits are
// wanted) the sum is RMS-normed by the model's norm instead and x stays as it is.
//
// HBM-bound: every operand is read once with 16-byte accesses and kept in registers between the passes; rows no vector
// width divides take a plain version that reads y again.
#include "ds_hip.h"

namespace {

// NT threads per token, E x 8 elements per thread
template <typename T, int NT, int E>
__global__ void __launch_bounds__(NT) post_norm_kernel(float* __restrict__ x, const T* __restrict__ y,
                                                       const float* __restrict__ w, const int* __restrict__ ids,
                                                       const T* __restrict__ embed, const int* __restrict__ rows,
                                                       const float* __restrict__ fw, float mult, T* __restrict__ out, int W,
                                                       float eps) {
  __shared__ float red[NT / 64];
  const int r = blockIdx.x, tid = threadIdx.x;
  const int64_t src = rows ? rows[r] : r;
  float* xr = x + src * W;
  if (embed) {
    const T* e = embed + (int64_t)ids[r] * W;
#pragma unroll
    for (int i = 0; i < E; ++i) {
      const int c = (tid + i * NT) * 8;
      if (c >= W) continue;
      float v[8];
      Vec8<T>::load(e + c, v);
      Vec8<float>::store(xr + c, v);
      Vec8<T>::store(out + (int64_t)r * W + c, v);
    }
    return;
  }
  float yv[E][8], xv[E][8], ss = 0.f;
#pragma unroll
  for (int i = 0; i < E; ++i) {
    const int c = (tid + i * NT) * 8, cc = c < W ? c : 0;
    Vec8<T>::load(y + src * W + cc, yv[i]);
    Vec8<float>::load(xr + cc, xv[i]);
    if (c < W) {
#pragma unroll
      for (int j = 0; j < 8; ++j) ss = fmaf(yv[i][j], yv[i][j], ss);
    }
  }
  const float rs = 1.f / sqrtf(block_sum(ss, red) / (float)W + eps);
  float s2 = 0.f;
#pragma unroll
  for (int i = 0; i < E; ++i) {
    const int c = (tid + i * NT) * 8;
    if (c >= W) continue;
    float g[8];
    Vec8<float>::load(w + c, g);
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      xv[i][j] = fmaf(yv[i][j] * rs, g[j], xv[i][j]);
      s2 = fmaf(xv[i][j], xv[i][j], s2);
    }
    if (!rows) {
      Vec8<float>::store(xr + c, xv[i]);
      Vec8<T>::store(out + (int64_t)r * W + c, xv[i]);
    }
  }
  if (!rows) return;
  const float r2 = mult / sqrtf(block_sum(s2, red) / (float)W + eps);
#pragma unroll
  for (int i = 0; i < E; ++i) {
    const int c = (tid + i * NT) * 8;
    if (c >= W) continue;
    float g[8];
    Vec8<float>::load(fw + c, g);
#pragma unroll
    for (int j = 0; j < 8; ++j) xv[i][j] *= r2 * g[j];
    Vec8<T>::store(out + (int64_t)r * W + c, xv[i]);
  }
}

// any width
template <typename T>
__global__ void __launch_bounds__(256) post_norm_any_kernel(float* __restrict__ x, const T* __restrict__ y,
                                                            const float* __restrict__ w, const int* __restrict__ ids,
                                                            const T* __restrict__ embed, const int* __restrict__ rows,
                                                            const float* __restrict__ fw, float mult, T* __restrict__ out,
                                                            int W, float eps) {
  __shared__ float red[4];
  const int r = blockIdx.x, tid = threadIdx.x;
  const int64_t src = rows ? rows[r] : r;
  float* xr = x + src * W;
  const T* yr = y + src * W;
  T* o = out + (int64_t)r * W;
  if (embed) {
    for (int c = tid; c < W; c += 256) {
      const float v = (float)embed[(int64_t)ids[r] * W + c];
      xr[c] = v;
      o[c] = (T)v;
    }
    return;
  }
  float ss = 0.f;
  for (int c = tid; c < W; c += 256) ss = fmaf((float)yr[c], (float)yr[c], ss);
  const float rs = 1.f / sqrtf(block_sum(ss, red) / (float)W + eps);
  float s2 = 0.f;
  for (int c = tid; c < W; c += 256) {
    const float v = fmaf((float)yr[c] * rs, w[c], xr[c]);
    s2 = fmaf(v, v, s2);
    if (!rows) {
      xr[c] = v;
      o[c] = (T)v;
    }
  }
  if (!rows) return;
  const float r2 = mult / sqrtf(block_sum(s2, red) / (float)W + eps);
  for (int c = tid; c < W; c += 256) o[c] = (T)(fmaf((float)yr[c] * rs, w[c], xr[c]) * r2 * fw[c]);
}

template <typename T>
int post_norm(float* x, const void* y, const float* w, const int* ids, const void* embed, const int* rows, int n,
              const float* fw, float mult, void* out, int W, float eps, hipStream_t st) {
#define GO(NT, E)                                                                                                    \
  hipLaunchKernelGGL((post_norm_kernel<T, NT, E>), dim3(n), dim3(NT), 0, st, x, (const T*)y, w, ids, (const T*)embed, \
                     rows, fw, mult, (T*)out, W, eps)
  if (W % 8 == 0 && W <= 16384) {
    if (W <= 512) GO(64, 1);
    else if (n <= 512 && W <= 4096) GO(512, 1);
    else if (n <= 512 && W <= 8192) GO(1024, 1);
    else if (n <= 512) GO(1024, 2);
    else if (W <= 2048) GO(256, 1);
    else if (W <= 4096) GO(256, 2);
    else if (W <= 8192) GO(256, 4);
    else GO(256, 8);
  } else {
    hipLaunchKernelGGL((post_norm_any_kernel<T>), dim3(n), dim3(256), 0, st, x, (const T*)y, w, ids, (const T*)embed, rows,
                       fw, mult, (T*)out, W, eps);
  }
#undef GO
  DS_CHECK_LAUNCH();
  return 0;
}

}  // namespace

extern "C" int ds_post_norm(float* x, const void* y, const float* w, const int* ids, const void* embed, const int* rows,
                            int n, const float* final_w, float mult, void* out, int W, float eps, int dtype,
                            hipStream_t st) {
  if (n <= 0) return 0;
  if (W <= 0 || (!y == !embed) || (y && !w) || (embed && !ids) || (rows && (!final_w || embed)))
    return (int)hipErrorInvalidValue;
  if (dtype == DS_F32) return post_norm<float>(x, y, w, ids, embed, rows, n, final_w, mult, out, W, eps, st);
  if (dtype == DS_BF16) return post_norm<bf16>(x, y, w, ids, embed, rows, n, final_w, mult, out, W, eps, st);
  return (int)hipErrorInvalidValue;
}
