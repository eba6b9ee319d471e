// What surrounds latent attention (latent_decode.hip, latent_prefill.hip), CDNA4 (gfx950).
//
// A token is cached as one row [latent c (R) | rotated key part (r)] shared by all heads. Keys and values are linear maps of
// c per head, so q . k = (W_uk^T q) . c: folding the map into the query leaves attention over the cached rows themselves.
//  * prepare: the down projection's row [query latent (Q, or none) | c (R) | key part (r)], which may be part of a wider one ->
//    normed query latent; c normed, the key part rotated to the token's position, both into the paged cache.
//  * head_linear: y[t, h] = W_h x[t, h] for every head, the maps of both directions; optionally the columns behind the map's
//    (the rotated part of the query) are rotated and carried over.
//  * rotate_tail: those columns in place, for queries that attend to expanded keys.
//  * gather: the cached rows of whole contexts laid end to end, operands of the expansion product.
// Angles are position * frequency in fp64, reduced to one turn, then fp32 sine and cosine, times a factor.
#include "ds_hip.h"

namespace {

struct Freq {
  const double* f;
  float mult;
};
__device__ __forceinline__ void turn_of(int pos, Freq freq, int i, float& c, float& s) {
  constexpr double TAU = 6.283185307179586476925286766559;
  const double a = (double)pos * freq.f[i];
  sincosf((float)(a - TAU * rint(a / TAU)), &s, &c);
  c *= freq.mult;
  s *= freq.mult;
}

// One wave per (token, part): part 0 the query latent, part 1 the cached row. V elements per access.
template <typename T, int V>
__global__ void __launch_bounds__(256) latent_prepare_kernel(
    const T* __restrict__ down, int64_t ld, const float* __restrict__ qw, const float* __restrict__ kvw, float eps,
    Freq freq, int half, const int* __restrict__ pos, const int* __restrict__ seq_ids,
    const int* __restrict__ bt, int max_blocks, T* __restrict__ lat, T* __restrict__ cq, int tokens, int Q, int R, int r,
    int BS) {
  const int lane = threadIdx.x & 63;
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  const int t = (int)(Q ? item >> 1 : item), part = Q ? (int)(item & 1) : 1;
  if (t >= tokens) return;
  const T* src = down + t * ld + (part ? Q : 0);
  const int W = part ? R : Q;
  const float* w = part ? kvw : qw;
  const int p = pos[t];
  T* dst = cq + (int64_t)t * Q;
  if (part) dst = lat + ((int64_t)bt[(int64_t)seq_ids[t] * max_blocks + p / BS] * BS + p % BS) * (R + r);
  float ss = 0.f;
  for (int c = lane * V; c < W; c += 64 * V) {
    float v[8];
    if constexpr (V == 8) Vec8<T>::load(src + c, v);
    else v[0] = (float)src[c];
#pragma unroll
    for (int j = 0; j < V; ++j) ss = fmaf(v[j], v[j], ss);
  }
  const float rs = 1.f / sqrtf(wave_sum(ss) / (float)W + eps);
  for (int c = lane * V; c < W; c += 64 * V) {
    if constexpr (V == 8) {
      float v[8], g[8];
      Vec8<T>::load(src + c, v);
      Vec8<float>::load(w + c, g);
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] *= rs * g[j];
      Vec8<T>::store(dst + c, v);
    } else {
      dst[c] = (T)((float)src[c] * rs * w[c]);
    }
  }
  if (!part) return;
  for (int i = lane; i < half; i += 64) {
    float co, si;
    turn_of(p, freq, i, co, si);
    const float u = (float)src[R + i], v = (float)src[R + half + i];
    dst[R + i] = (T)(u * co - v * si);
    dst[R + half + i] = (T)(v * co + u * si);
  }
  for (int i = 2 * half + lane; i < r; i += 64) dst[R + i] = src[R + i];
}

// Item j of the columns behind the map's: pair (j, half + j) turned, or a single column carried over
template <typename T>
__device__ __forceinline__ void rotate_one(const T* s, T* d, int j, int half, int p, Freq freq) {
  if (j < half) {
    float co, si;
    turn_of(p, freq, j, co, si);
    const float u = (float)s[j], v = (float)s[half + j];
    d[j] = (T)(u * co - v * si);
    d[half + j] = (T)(v * co + u * si);
  } else {
    d[half + j] = s[half + j];
  }
}

// ... of all heads of a token, by a workgroup
template <typename T>
__device__ __forceinline__ void rotate_heads(const T* src, int64_t sh, T* dst, int64_t dh, int H, int r, int half, int p,
                                             Freq freq) {
  const int per = r - half;
  for (int i = threadIdx.x; i < H * per; i += blockDim.x)
    rotate_one(src + i / per * sh, dst + i / per * dh, i % per, half, p, freq);
}

template <typename T>
__global__ void __launch_bounds__(256) rotate_tail_kernel(T* __restrict__ q, int64_t ld, int64_t row, int d, int r, int H,
                                                          Freq freq, int half, const int* __restrict__ pos) {
  __shared__ float cs[2][256];
  const int t = blockIdx.x, p = pos[t];
  T* x = q + t * ld + d;
  if (half <= 256) {  // one sine and cosine per pair, shared by the heads
    for (int i = threadIdx.x; i < half; i += 256) turn_of(p, freq, i, cs[0][i], cs[1][i]);
    __syncthreads();
    for (int i = threadIdx.x; i < H * half; i += 256) {
      const int h = i / half, j = i % half;
      T* s = x + h * row;
      const float co = cs[0][j], si = cs[1][j], u = (float)s[j], v = (float)s[half + j];
      s[j] = (T)(u * co - v * si);
      s[half + j] = (T)(v * co + u * si);
    }
  } else {
    rotate_heads(x, row, x, row, H, r, half, p, freq);
  }
}

struct HeadArgs {
  const void* x;     // [T, H, xrow], K columns used, ldx elements from token to token
  const void* w;     // [H, N, K]
  void* y;           // [T, H, yrow]
  int T, H, N, K, xrow, yrow;
  int r, half;       // columns K .. K + r of x go to N .. N + r of y, the first 2 half of them rotated
  Freq freq;
  const int* pos;
  int64_t ldx;
};

// TT x 16 tokens, 64 output columns (16 per wave) of one head: W rows as the A operand, tokens as B
template <int TT>
__global__ void __launch_bounds__(256) head_linear_mfma_kernel(HeadArgs a) {
  const int h = blockIdx.y, lane = threadIdx.x & 63, wid = threadIdx.x >> 6, l16 = lane & 15, q4 = lane >> 4;
  const int t0 = blockIdx.z * 16 * TT, ntiles = (a.N + 63) / 64;
  if ((int)blockIdx.x >= ntiles) {
    const int per = a.r - a.half, nt = min(16 * TT, a.T - t0);  // pairs and single columns of a token
    for (int i = threadIdx.x; i < nt * per; i += 256) {
      const int t = t0 + i / per;
      rotate_one((const bf16*)a.x + t * a.ldx + h * a.xrow + a.K, (bf16*)a.y + ((int64_t)t * a.H + h) * a.yrow + a.N,
                 i % per, a.half, a.pos[t], a.freq);
    }
    return;
  }
  const int n0 = blockIdx.x * 64 + wid * 16;
  if (n0 >= a.N) return;
  const bf16* wr = (const bf16*)a.w + ((int64_t)h * a.N + min(n0 + l16, a.N - 1)) * a.K;
  const bf16* xr[TT];
#pragma unroll
  for (int i = 0; i < TT; ++i)
    xr[i] = (const bf16*)a.x + min(t0 + 16 * i + l16, a.T - 1) * a.ldx + h * a.xrow;
  f32x4 acc[TT];
#pragma unroll
  for (int i = 0; i < TT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int full = a.K / 32;
  for (int s = 0; s < full; ++s) {
    const bf16x8 wv = *reinterpret_cast<const bf16x8*>(wr + 32 * s + 8 * q4);
#pragma unroll
    for (int i = 0; i < TT; ++i)
      acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv, *reinterpret_cast<const bf16x8*>(xr[i] + 32 * s + 8 * q4),
                                                       acc[i], 0, 0, 0);
  }
  if (a.K % 32) {
    const int k = 32 * full + 8 * q4;
    bf16x8 z;
#pragma unroll
    for (int j = 0; j < 8; ++j) z[j] = (bf16)0.f;
    const bf16x8 wv = k < a.K ? *reinterpret_cast<const bf16x8*>(wr + k) : z;
#pragma unroll
    for (int i = 0; i < TT; ++i)
      acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv, k < a.K ? *reinterpret_cast<const bf16x8*>(xr[i] + k) : z, acc[i],
                                                       0, 0, 0);
  }
#pragma unroll
  for (int i = 0; i < TT; ++i) {
    const int t = t0 + 16 * i + l16, n = n0 + 4 * q4;
    if (t >= a.T) continue;
    bf16* y = (bf16*)a.y + ((int64_t)t * a.H + h) * a.yrow + n;
    bf16x4 o;
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = (bf16)acc[i][j];
    if (n + 3 < a.N && a.yrow % 4 == 0) {
      *reinterpret_cast<bf16x4*>(y) = o;
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (n + j < a.N) y[j] = o[j];
    }
  }
}

// any sizes: a workgroup per (token, head), a thread per output column
template <typename T>
__global__ void __launch_bounds__(256) head_linear_any_kernel(HeadArgs a) {
  const int t = blockIdx.x, h = blockIdx.y;
  const T* x = (const T*)a.x + t * a.ldx + h * a.xrow;
  T* y = (T*)a.y + ((int64_t)t * a.H + h) * a.yrow;
  for (int n = threadIdx.x; n < a.N; n += 256) {
    const T* w = (const T*)a.w + ((int64_t)h * a.N + n) * a.K;
    float s = 0.f;
    for (int k = 0; k < a.K; ++k) s = fmaf((float)w[k], (float)x[k], s);
    y[n] = (T)s;
  }
  if (a.r) rotate_heads(x + a.K, 0, y + a.N, 0, 1, a.r, a.half, a.pos[t], a.freq);
}

// one wave per context row of 16-byte pieces
__global__ void __launch_bounds__(256) latent_gather_kernel(const bf16* __restrict__ lat, const int* __restrict__ bt,
                                                            int max_blocks, const int* __restrict__ offs,
                                                            const int* __restrict__ first_keys, int first,
                                                            int nseq, bf16* __restrict__ ctx, int64_t total, int pad,
                                                            int row, int BS) {
  const int64_t i = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (i >= total + pad) return;
  if (i >= total) {
    for (int c = (threadIdx.x & 63) * 8; c < row; c += 512) {
      bf16x8 z;
#pragma unroll
      for (int j = 0; j < 8; ++j) z[j] = (bf16)0.f;
      *reinterpret_cast<bf16x8*>(ctx + i * row + c) = z;
    }
    return;
  }
  int s = 0;
  while (s + 1 < nseq && i >= offs[s + 1]) ++s;
  const int p = (int)(i - offs[s]) + (first_keys ? first_keys[s] : 0);
  const bf16* src = lat + ((int64_t)bt[(int64_t)(first + s) * max_blocks + p / BS] * BS + p % BS) * row;
  for (int c = (threadIdx.x & 63) * 8; c < row; c += 512)
    *reinterpret_cast<bf16x8*>(ctx + i * row + c) = *reinterpret_cast<const bf16x8*>(src + c);
}

}  // namespace

// down: rows ld elements apart; Q 0: no query latent (qw, cq unused); cosine and sine times mult
extern "C" int ds_latent_prepare(const void* down, int64_t ld, const float* qw, const float* kvw, float eps, const double* freq,
                                 float mult, int half,
                                 const int* pos, const int* seq_ids, const int* bt, int max_blocks, void* lat, void* cq,
                                 int tokens, int Q, int R, int r, int BS, int dtype, hipStream_t st) {
  if (tokens <= 0) return 0;
  if (Q < 0 || (Q && (!qw || !cq)) || ld < (int64_t)Q + R + r || R <= 0 || r < 0 || half < 0 || 2 * half > r || BS <= 0 || max_blocks <= 0) return (int)hipErrorInvalidValue;
  const bool vec = Q % 8 == 0 && R % 8 == 0 && r % 8 == 0 && ld % 8 == 0 && ((uintptr_t)down & 15) == 0;
  const int64_t items = (int64_t)tokens * (Q ? 2 : 1);
#define GO(T, V)                                                                                                      \
  hipLaunchKernelGGL((latent_prepare_kernel<T, V>), dim3((unsigned)((items + 3) / 4)), dim3(256), 0, st, (const T*)down, ld, qw, kvw, \
                     eps, Freq{freq, mult}, half, pos, seq_ids, bt, max_blocks, (T*)lat, (T*)cq, tokens, Q, R, r, BS)
  if (dtype == DS_F32 && vec) GO(float, 8);
  else if (dtype == DS_F32) GO(float, 1);
  else if (dtype == DS_BF16 && vec) GO(bf16, 8);
  else if (dtype == DS_BF16) GO(bf16, 1);
  else return (int)hipErrorInvalidValue;
#undef GO
  DS_CHECK_LAUNCH();
  return 0;
}

// ld: elements from token to token
extern "C" int ds_rotate_tail(void* q, int64_t ld, int tokens, int H, int row, int r, const double* freq, float mult, int half,
                              const int* pos, int dtype, hipStream_t st) {
  if (tokens <= 0 || half <= 0) return 0;
  if (H <= 0 || r > row || 2 * half > r || ld < (int64_t)H * row) return (int)hipErrorInvalidValue;
  if (dtype == DS_F32)
    hipLaunchKernelGGL((rotate_tail_kernel<float>), dim3(tokens), dim3(256), 0, st, (float*)q, ld, (int64_t)row, row - r, r,
                       H, Freq{freq, mult}, half, pos);
  else if (dtype == DS_BF16)
    hipLaunchKernelGGL((rotate_tail_kernel<bf16>), dim3(tokens), dim3(256), 0, st, (bf16*)q, ld, (int64_t)row, row - r, r,
                       H, Freq{freq, mult}, half, pos);
  else return (int)hipErrorInvalidValue;
  DS_CHECK_LAUNCH();
  return 0;
}

// x [T, H, xrow] (ldx elements from token to token), w [H, N, K], y [T, H, yrow]; r > 0: columns K .. K + r of x, rotated, behind the N of y
extern "C" int ds_head_linear(const void* x, const void* w, void* y, int T, int H, int N, int K, int xrow, int yrow, int r,
                              int64_t ldx, int half, const double* freq, float mult, const int* pos, int dtype, hipStream_t st) {
  if (T <= 0) return 0;
  if (H <= 0 || H > 65535 || N <= 0 || K <= 0 || xrow < K + r || yrow < N + r || 2 * half > r || (r && (!freq || !pos)) ||
      ldx < (int64_t)H * xrow)
    return (int)hipErrorInvalidValue;
  const HeadArgs a{x, w, y, T, H, N, K, xrow, yrow, r, half, Freq{freq, mult}, pos, ldx};
  if (dtype == DS_BF16 && K % 8 == 0 && xrow % 8 == 0 && ldx % 8 == 0 && (((uintptr_t)x | (uintptr_t)w) & 15) == 0 && (T + 15) / 16 <= 65535) {
    const int tiles = (N + 63) / 64 + (r ? 1 : 0);
    if (T <= 16) hipLaunchKernelGGL((head_linear_mfma_kernel<1>), dim3(tiles, H, 1), dim3(256), 0, st, a);
    else if (T <= 64) hipLaunchKernelGGL((head_linear_mfma_kernel<2>), dim3(tiles, H, (T + 31) / 32), dim3(256), 0, st, a);
    else hipLaunchKernelGGL((head_linear_mfma_kernel<4>), dim3(tiles, H, (T + 63) / 64), dim3(256), 0, st, a);
  } else if (dtype == DS_BF16) {
    hipLaunchKernelGGL((head_linear_any_kernel<bf16>), dim3(T, H), dim3(256), 0, st, a);
  } else if (dtype == DS_F32) {
    hipLaunchKernelGGL((head_linear_any_kernel<float>), dim3(T, H), dim3(256), 0, st, a);
  } else {
    return (int)hipErrorInvalidValue;
  }
  DS_CHECK_LAUNCH();
  return 0;
}

// contexts of sequences first .. first + nseq from their first keys on (null: 0), offs [nseq + 1] their places in ctx
// [total + pad, row] (bf16), whose last `pad` rows become zero
extern "C" int ds_latent_gather(const void* lat, const int* bt, int max_blocks, const int* offs, const int* first_keys, int first, int nseq, void* ctx,
                                int64_t total, int pad, int row, int BS, hipStream_t st) {
  if (total <= 0) return 0;
  if (row <= 0 || row % 8 || BS <= 0 || max_blocks <= 0 || nseq <= 0) return (int)hipErrorInvalidValue;
  hipLaunchKernelGGL(latent_gather_kernel, dim3((unsigned)((total + pad + 3) / 4)), dim3(256), 0, st, (const bf16*)lat, bt,
                     max_blocks, offs, first_keys, first, nseq, (bf16*)ctx, total, pad, row, BS);
  DS_CHECK_LAUNCH();
  return 0;
}
