// Plain fp32 residual with RMS norms on the sublayers' inputs and, optionally, on their gated outputs, CDNA4 (gfx950). One launch
// per sublayer boundary:
//   1. y: a sublayer's output, or sum_k w[t, k] y[row(t, k)] + base[t] (the weighted outputs of a token's experts, and of one
//      that every token takes);
//   2. (POST) y <- sigmoid(gate + gate bias) y, if there is a gate, then y <- y / rms(y) * post weight;
//   3. x <- x + y, or, at the start of the model, x <- the token's embedding row times a constant;
//   4. the next sublayer's input x / rms(x) * w in the storage type (without w: x itself).
// With a row list (the rows whose logits are wanted) only those rows are normed and x stays as it is.
//
// HBM-bound: every operand is read once with 16-byte accesses, the row stays in registers between the passes; widths that are
// no multiple of 8 take a plain version that goes over the row again.
#include "ds_hip.h"

namespace {

struct PreArgs {
  float* x;            // [T, W]
  const void* y;       // [T, W] or [T * K, W]
  const float* yw;     // [T, K] or null
  const int* yrow;     // [T, K]: rows of y; null: t * K + k
  const void* base;    // [T, W] or null (with yw)
  int K;
  const float* post;   // [W] or null
  const void* gate;    // [T, W] or null (with post), rows ldg apart
  const float* gate_b; // [W]
  int64_t ldg;
  const int* ids;      // [T]
  const void* embed;   // [V, W]
  float mult;          // of the embedding
  const int* rows;
  const float* w;      // [W] or null
  void* out;
  int W;
  float eps;
};

// What the sublayer before leaves for columns c .. c + 7 of token t
template <typename T>
__device__ __forceinline__ void added(const PreArgs& a, int64_t t, int c, float (&v)[8]) {
  const T* y = (const T*)a.y;
  if (!a.yw) {
    Vec8<T>::load(y + t * a.W + c, v);
    return;
  }
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] = 0.f;
#pragma unroll 4
  for (int k = 0; k < a.K; ++k) {
    const int64_t e = t * a.K + k, r = a.yrow ? a.yrow[e] : e;
    float u[8];
    Vec8<T>::load(y + r * a.W + c, u);
    const float g = a.yw[e];
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = fmaf(g, u[j], v[j]);
  }
  if (a.base) {
    float u[8];
    Vec8<T>::load((const T*)a.base + t * a.W + c, u);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] += u[j];
  }
}

__device__ __forceinline__ float gated(float y, float g) { return y / (1.f + expf(-g)); }

// NT threads per token, E x 8 elements per thread
template <typename T, int NT, int E, bool POST>
__global__ void __launch_bounds__(NT) pre_norm_kernel(PreArgs a) {
  __shared__ float red[NT / 64];
  const int r = blockIdx.x, tid = threadIdx.x, W = a.W;
  const int64_t src = a.rows ? a.rows[r] : r;
  float* xr = a.x + src * W;
  float xv[E][8], ss = 0.f;
  float yv[POST ? E : 1][8], post[POST ? E : 1][8];
  if constexpr (POST) {
    float sy = 0.f;
#pragma unroll
    for (int i = 0; i < E; ++i) {
      const int c = (tid + i * NT) * 8;
      if (c >= W) continue;
      float g[8], b[8];
      if (a.gate) {
        Vec8<T>::load((const T*)a.gate + src * a.ldg + c, g);
        Vec8<float>::load(a.gate_b + c, b);
      }
      Vec8<float>::load(a.post + c, post[i]);
      Vec8<float>::load(xr + c, xv[i]);
      added<T>(a, src, c, yv[i]);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        if (a.gate) yv[i][j] = gated(yv[i][j], g[j] + b[j]);
        sy = fmaf(yv[i][j], yv[i][j], sy);
      }
    }
    const float ry = 1.f / sqrtf(block_sum(sy, red) / (float)W + a.eps);
#pragma unroll
    for (int i = 0; i < E; ++i)
#pragma unroll
      for (int j = 0; j < 8; ++j) yv[i][j] *= ry * post[i][j];
  }
#pragma unroll
  for (int i = 0; i < E; ++i) {
    const int c = (tid + i * NT) * 8;
    if (c >= W) continue;
    if constexpr (POST) {
#pragma unroll
      for (int j = 0; j < 8; ++j) xv[i][j] += yv[i][j];
    } else if (a.embed) {
      Vec8<T>::load((const T*)a.embed + (int64_t)a.ids[r] * W + c, xv[i]);
#pragma unroll
      for (int j = 0; j < 8; ++j) xv[i][j] *= a.mult;
    } else {
      float v[8];
      Vec8<float>::load(xr + c, xv[i]);
      added<T>(a, src, c, v);
#pragma unroll
      for (int j = 0; j < 8; ++j) xv[i][j] += v[j];
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) ss = fmaf(xv[i][j], xv[i][j], ss);
    if (!a.rows) Vec8<float>::store(xr + c, xv[i]);
    if (!a.w) Vec8<T>::store((T*)a.out + (int64_t)r * W + c, xv[i]);
  }
  if (!a.w) return;
  const float rs = 1.f / sqrtf(block_sum(ss, red) / (float)W + a.eps);
#pragma unroll
  for (int i = 0; i < E; ++i) {
    const int c = (tid + i * NT) * 8;
    if (c >= W) continue;
    float g[8];
    Vec8<float>::load(a.w + c, g);
#pragma unroll
    for (int j = 0; j < 8; ++j) xv[i][j] *= rs * g[j];
    Vec8<T>::store((T*)a.out + (int64_t)r * W + c, xv[i]);
  }
}

// any width
template <typename T>
__global__ void __launch_bounds__(256) pre_norm_any_kernel(PreArgs a) {
  __shared__ float red[4];
  const int r = blockIdx.x, tid = threadIdx.x, W = a.W;
  const int64_t src = a.rows ? a.rows[r] : r;
  const T* y = (const T*)a.y;
  float* xr = a.x + src * W;
  auto added_one = [&](int c) {
    float v = 0.f;
    if (!a.yw) {
      v = (float)y[src * W + c];
    } else {
      for (int k = 0; k < a.K; ++k) {
        const int64_t e = src * a.K + k;
        v = fmaf(a.yw[e], (float)y[(a.yrow ? a.yrow[e] : e) * W + c], v);
      }
      if (a.base) v += (float)((const T*)a.base)[src * W + c];
    }
    return a.gate ? gated(v, (float)((const T*)a.gate)[src * a.ldg + c] + a.gate_b[c]) : v;
  };
  float ry = 1.f;
  if (a.post) {
    float sy = 0.f;
    for (int c = tid; c < W; c += 256) {
      const float v = added_one(c);
      sy = fmaf(v, v, sy);
    }
    ry = 1.f / sqrtf(block_sum(sy, red) / (float)W + a.eps);
  }
  auto sum = [&](int c) {
    if (a.embed) return (float)((const T*)a.embed)[(int64_t)a.ids[r] * W + c] * a.mult;
    return xr[c] + added_one(c) * (a.post ? ry * a.post[c] : 1.f);
  };
  float ss = 0.f;
  for (int c = tid; c < W; c += 256) {
    const float v = sum(c);
    ss = fmaf(v, v, ss);
    if (!a.rows) xr[c] = v;
  }
  const float rs = 1.f / sqrtf(block_sum(ss, red) / (float)W + a.eps);
  for (int c = tid; c < W; c += 256)  // (each thread re-reads what it wrote)
    ((T*)a.out)[(int64_t)r * W + c] = (T)((a.rows ? sum(c) : xr[c]) * (a.w ? rs * a.w[c] : 1.f));
}

template <typename T>
int pre_norm(const PreArgs& a, int n, hipStream_t st) {
#define GO(NT, E)                                                                                 {                                                                                                 if (a.post) hipLaunchKernelGGL((pre_norm_kernel<T, NT, E, true>), dim3(n), dim3(NT), 0, st, a);     else hipLaunchKernelGGL((pre_norm_kernel<T, NT, E, false>), dim3(n), dim3(NT), 0, st, a);     }
  const int W = a.W;
  if (W % 8 == 0 && W <= 16384 && a.ldg % 8 == 0 && ((uintptr_t)a.gate & 15) == 0) {
    if (W <= 512) GO(64, 1)
    else if (n <= 512 && W <= 4096) GO(512, 1)
    else if (n <= 512 && W <= 8192) GO(1024, 1)
    else if (n <= 512) GO(1024, 2)
    else if (W <= 2048) GO(256, 1)
    else if (W <= 4096) GO(256, 2)
    else if (W <= 8192) GO(256, 4)
    else GO(256, 8)
  } else {
    hipLaunchKernelGGL((pre_norm_any_kernel<T>), dim3(n), dim3(256), 0, st, a);
  }
#undef GO
  DS_CHECK_LAUNCH();
  return 0;
}

}  // namespace

// y [T, W] (yw null), or y [.., W] with yw [T, K], optionally yrow [T, K] and base [T, W]; or ids and embed, times mult. post:
// y's norm, with gate [T, W] (rows ldg apart) and gate_b or without. w null: no norm of the sum. -> out [n, W]
extern "C" int ds_pre_norm(float* x, const void* y, const float* yw, const int* yrow, const void* base, int K, const float* post,
                           const void* gate, int64_t ldg, const float* gate_b, const int* ids, const void* embed, float mult,
                           const int* rows, int n, const float* w, void* out, int W, float eps, int dtype, hipStream_t st) {
  if (n <= 0) return 0;
  if (W <= 0 || (!y == !embed) || (embed && (!ids || rows || post)) || (yw && K <= 0) || (gate && (!post || !gate_b || ldg < W)) ||
      (base && !yw))
    return (int)hipErrorInvalidValue;
  const PreArgs a{x, y, yw, yrow, base, K, post, gate, gate_b, gate ? ldg : 0, ids, embed, mult, rows, w, out, W, eps};
  if (dtype == DS_F32) return pre_norm<float>(a, n, st);
  if (dtype == DS_BF16) return pre_norm<bf16>(a, n, st);
  return (int)hipErrorInvalidValue;
}
