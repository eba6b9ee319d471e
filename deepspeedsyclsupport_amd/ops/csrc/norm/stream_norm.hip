// Multi-stream residual (hyper-connections) fused with the pre-norm of the next sublayer, CDNA4 (gfx950).
//
// The residual is S streams per token, x [T, S, W] in fp32. One launch per sublayer boundary
//   1. finishes the sublayer before it:  x_t <- sum_s mix[s, t] * x_s + m * out[t] * y      (all t from the old x)
//      or, at the start of the model, sets every stream to the token's embedding row;
//   2. forms the input of the sublayer after it:  u = sum_s in[s] * x_s;
//   3. normalises it: (u - mean) / sqrt(var + eps) * w, the variance over squared deviations (second pass over u in LDS).
// A plain residual is the special case S = 1, mix = in = out = 1. With a row list only those rows are normalised and
// the streams are not written back (the rows whose logits are wanted, after the last sublayer).
//
// HBM-bound: per token the streams are read and written once, y read once and the normed row written once; one
// workgroup per token, 16-byte accesses, u kept in LDS between the passes.
#include "ds_hip.h"

namespace {

template <typename T, int V>
__device__ __forceinline__ void ldv(const T* p, float (&v)[V]) {
  if constexpr (V == 1) {
    v[0] = (float)p[0];
  } else if constexpr (sizeof(T) == 4) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = a[i];
  } else {
    const bf16x4 a = *reinterpret_cast<const bf16x4*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = (float)a[i];
  }
}
template <typename T, int V>
__device__ __forceinline__ void stv(T* p, const float (&v)[V]) {
  if constexpr (V == 1) {
    p[0] = (T)v[0];
  } else if constexpr (sizeof(T) == 4) {
    f32x4 a;
#pragma unroll
    for (int i = 0; i < 4; ++i) a[i] = v[i];
    *reinterpret_cast<f32x4*>(p) = a;
  } else {
    bf16x4 a;
#pragma unroll
    for (int i = 0; i < 4; ++i) a[i] = (bf16)v[i];
    *reinterpret_cast<bf16x4*>(p) = a;
  }
}

// NT threads per token: 256, or 1024 when there are too few tokens to fill the chip (latency counts then)
template <typename T, int S, int V, int NT>
__global__ void __launch_bounds__(NT) stream_norm_kernel(
    float* __restrict__ x, const T* __restrict__ y, const int* __restrict__ ids, const T* __restrict__ embed,
    const int* __restrict__ rows, const float* __restrict__ mix, const float* __restrict__ out, float m,
    const float* __restrict__ in, const float* __restrict__ w, T* __restrict__ normed, int W, float eps) {
  extern __shared__ __attribute__((aligned(16))) float u[];  // [W] + reduction scratch
  float* red = u + ((W + 3) & ~3);
  const int r = blockIdx.x, tid = threadIdx.x;
  const int64_t src = rows ? rows[r] : r;
  float* xr = x + src * S * W;
  float cm[S][S], co[S], ci[S];
#pragma unroll
  for (int s = 0; s < S; ++s) {
    ci[s] = in ? in[s] : 1.f;
    co[s] = y ? m * out[s] : 0.f;
#pragma unroll
    for (int t = 0; t < S; ++t) cm[s][t] = y ? mix[s * S + t] : 0.f;
  }
  float sum = 0.f;
  for (int c = tid * V; c < W; c += NT * V) {
    float xs[S][V], xn[S][V], uu[V];
    if (embed) {
      float e[V];
      ldv<T, V>(embed + (int64_t)ids[r] * W + c, e);
#pragma unroll
      for (int s = 0; s < S; ++s)
#pragma unroll
        for (int i = 0; i < V; ++i) xn[s][i] = e[i];
    } else {
#pragma unroll
      for (int s = 0; s < S; ++s) ldv<float, V>(xr + (int64_t)s * W + c, xs[s]);
      if (y) {
        float yv[V];
        ldv<T, V>(y + src * W + c, yv);
#pragma unroll
        for (int t = 0; t < S; ++t)
#pragma unroll
          for (int i = 0; i < V; ++i) {
            float a = co[t] * yv[i];
#pragma unroll
            for (int s = 0; s < S; ++s) a = fmaf(cm[s][t], xs[s][i], a);
            xn[t][i] = a;
          }
      } else {
#pragma unroll
        for (int s = 0; s < S; ++s)
#pragma unroll
          for (int i = 0; i < V; ++i) xn[s][i] = xs[s][i];
      }
    }
    if (!rows && (embed || y)) {
#pragma unroll
      for (int s = 0; s < S; ++s) stv<float, V>(xr + (int64_t)s * W + c, xn[s]);
    }
#pragma unroll
    for (int i = 0; i < V; ++i) {
      float a = 0.f;
#pragma unroll
      for (int s = 0; s < S; ++s) a = fmaf(ci[s], xn[s][i], a);
      uu[i] = a;
      sum += a;
    }
    stv<float, V>(u + c, uu);
  }
  if (!normed) return;
  const float mean = block_sum(sum, red) / (float)W;
  float ss = 0.f;
  for (int c = tid * V; c < W; c += NT * V) {
    float uu[V];
    ldv<float, V>(u + c, uu);  // each thread re-reads what it wrote
#pragma unroll
    for (int i = 0; i < V; ++i) ss = fmaf(uu[i] - mean, uu[i] - mean, ss);
  }
  const float rs = 1.f / sqrtf(block_sum(ss, red) / (float)W + eps);
  for (int c = tid * V; c < W; c += NT * V) {
    float uu[V], ww[V];
    ldv<float, V>(u + c, uu);
    ldv<float, V>(w + c, ww);
#pragma unroll
    for (int i = 0; i < V; ++i) uu[i] = (uu[i] - mean) * rs * ww[i];
    stv<T, V>(normed + (int64_t)r * W + c, uu);
  }
}

template <typename T, int S>
int launch(float* x, const void* y, const int* ids, const void* embed, const int* rows, int nrows, const float* mix,
           const float* out, float m, const float* in, const float* w, void* normed, int W, float eps, hipStream_t st) {
  const size_t lds = (size_t)(((W + 3) & ~3) + 16) * sizeof(float);
#define GO(V, NT)                                                                                                   \
  hipLaunchKernelGGL((stream_norm_kernel<T, S, V, NT>), dim3(nrows), dim3(NT), lds, st, x, (const T*)y, ids,            \
                     (const T*)embed, rows, mix, out, m, in, w, (T*)normed, W, eps)
  const bool wide = nrows <= 512 && W >= 2048;
  if (W % 4 == 0 && wide) GO(4, 1024);
  else if (W % 4 == 0) GO(4, 256);
  else GO(1, 256);
#undef GO
  DS_CHECK_LAUNCH();
  return 0;
}

template <typename T>
int by_streams(int S, float* x, const void* y, const int* ids, const void* embed, const int* rows, int nrows,
               const float* mix, const float* out, float m, const float* in, const float* w, void* normed, int W,
               float eps, hipStream_t st) {
#define CASE(N) \
  case N: return launch<T, N>(x, y, ids, embed, rows, nrows, mix, out, m, in, w, normed, W, eps, st);
  switch (S) {
    CASE(1) CASE(2) CASE(3) CASE(4) CASE(5) CASE(6) CASE(7) CASE(8)
    default: return (int)hipErrorInvalidValue;
  }
#undef CASE
}

}  // namespace

extern "C" int ds_stream_norm(float* x, const void* y, const int* ids, const void* embed, const int* rows, int nrows,
                              int S, const float* mix, const float* out, float m, const float* in, const float* w,
                              void* normed, int W, float eps, int dtype, hipStream_t st) {
  if (nrows <= 0) return 0;
  if (W <= 0 || W > 15360 || (y && embed) || (y && (!mix || !out)) || (embed && !ids)) return (int)hipErrorInvalidValue;
  if (dtype == DS_F32)
    return by_streams<float>(S, x, y, ids, embed, rows, nrows, mix, out, m, in, w, normed, W, eps, st);
  if (dtype == DS_BF16)
    return by_streams<bf16>(S, x, y, ids, embed, rows, nrows, mix, out, m, in, w, normed, W, eps, st);
  return (int)hipErrorInvalidValue;
}
