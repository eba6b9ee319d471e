// QKV epilogue of attention layers that norm the query and key projections as a whole and rotate part of every head, CDNA4
// (gfx950); and the angle tables that such layers share.
//
//  * rope_table: cos and sin of position * frequency, times a factor, for every token of the batch. The angle is taken in fp64 and reduced to
//    one turn before the fp32 functions, so far positions lose nothing. One table serves all heads of all layers with these
//    frequencies.
//  * qk_rope_append: one workgroup per token. A projection row [q | k | v] (it may be part of a wider one) gets its biases;
//    q and k are divided by the root mean square over all their heads, times a weight; pairs (i, i + half) of each head's
//    first 2 half columns are turned; q is written out, k and v (times a factor) go straight into the paged cache, whose key
//    and value rows may differ in width. The row waits in LDS between the sums of squares and the rotation.
#include "ds_hip.h"

namespace {

__global__ void __launch_bounds__(256) rope_table_kernel(const int* __restrict__ pos, const double* __restrict__ freq,
                                                         f32x2* __restrict__ cs, int64_t items, int half, float mult) {
  constexpr double TAU = 6.283185307179586476925286766559;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < items; i += (int64_t)gridDim.x * 256) {
    const double a = (double)pos[i / half] * freq[i % half];
    float c, s;
    sincosf((float)(a - TAU * rint(a / TAU)), &s, &c);
    cs[i] = f32x2{c * mult, s * mult};
  }
}

template <typename T, int V>
__device__ __forceinline__ void ldx(const T* p, float (&v)[V]) {
  if constexpr (V == 8) Vec8<T>::load(p, v);
  else v[0] = (float)p[0];
}
template <typename T, int V>
__device__ __forceinline__ void stx(T* p, const float (&v)[V]) {
  if constexpr (V == 8) Vec8<T>::store(p, v);
  else p[0] = (T)v[0];
}

// V elements per access: 8 where every width is a multiple of it
template <typename T, int V>
__global__ void __launch_bounds__(256) qk_rope_append_kernel(
    const T* __restrict__ qkv, int64_t ld, const float* __restrict__ bias, const float* __restrict__ qw,
    const float* __restrict__ kw, float eps, const float* __restrict__ cs, int half, float vmult,
    const int* __restrict__ pos, const int* __restrict__ seq_ids, const int* __restrict__ block_table, int max_blocks,
    T* __restrict__ q_out, T* __restrict__ kc, T* __restrict__ vc, int H, int G, int dk, int dv, int BS) {
  extern __shared__ __attribute__((aligned(16))) float xs[];  // [(H + G) dk]
  __shared__ float red[4];
  const int t = blockIdx.x, tid = threadIdx.x, nq = H * dk, nqk = nq + G * dk;
  const T* row = qkv + t * ld;
  const int p = pos[t];
  const int64_t blk = block_table[(int64_t)seq_ids[t] * max_blocks + p / BS];
  const int off = p % BS;
  float sq = 0.f, sk = 0.f;
  for (int c = tid * V; c < nqk; c += 256 * V) {
    float x[V], b[V];
    ldx<T, V>(row + c, x);
    if (bias) {
      ldx<float, V>(bias + c, b);
#pragma unroll
      for (int j = 0; j < V; ++j) x[j] += b[j];
    }
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < V; ++j) s = fmaf(x[j], x[j], s);
    stx<float, V>(xs + c, x);
    if (c < nq) sq += s;
    else sk += s;
  }
  for (int c = tid * V; c < G * dv; c += 256 * V) {
    float x[V], b[V];
    ldx<T, V>(row + nqk + c, x);
    if (bias) {
      ldx<float, V>(bias + nqk + c, b);
#pragma unroll
      for (int j = 0; j < V; ++j) x[j] += b[j];
    }
#pragma unroll
    for (int j = 0; j < V; ++j) x[j] *= vmult;
    stx<T, V>(vc + ((blk * G + c / dv) * BS + off) * dv + c % dv, x);
  }
  sq = block_sum(sq, red);
  sk = block_sum(sk, red);
  const float rq = qw ? 1.f / sqrtf(sq / (float)nq + eps) : 1.f, rk = kw ? 1.f / sqrtf(sk / (float)(nqk - nq) + eps) : 1.f;
  const float* ct = cs + (int64_t)t * half * 2;
  for (int c = tid * V; c < nqk; c += 256 * V) {
    const bool isq = c < nq;
    const int cc = isq ? c : c - nq, h = cc / dk, d = cc % dk;
    const float r = isq ? rq : rk;
    const float* w = isq ? qw : kw;
    float x[V], g[V];
    ldx<float, V>(xs + c, x);
    if (w) {
      ldx<float, V>(w + cc, g);
#pragma unroll
      for (int j = 0; j < V; ++j) x[j] *= r * g[j];
    }
    if (d < 2 * half) {  // (V divides half)
      const bool lo = d < half;
      const int o = lo ? half : -half;
      float y[V];
      ldx<float, V>(xs + c + o, y);
      if (w) {
        ldx<float, V>(w + cc + o, g);
#pragma unroll
        for (int j = 0; j < V; ++j) y[j] *= r * g[j];
      }
      const float* a = ct + 2 * (lo ? d : d - half);
#pragma unroll
      for (int j = 0; j < V; ++j) x[j] = x[j] * a[2 * j] + (lo ? -y[j] : y[j]) * a[2 * j + 1];
    }
    stx<T, V>(isq ? q_out + (int64_t)t * nq + c : kc + ((blk * G + h) * BS + off) * dk + d, x);
  }
}

constexpr int MAX_LDS = 144 * 1024;

template <typename T, int V>
int launch(const void* qkv, int64_t ld, const float* bias, const float* qw, const float* kw, float eps, const float* cs,
           int half, float vmult, const int* pos, const int* seq_ids, const int* bt, int max_blocks, void* q, void* kc,
           void* vc, int tokens, int H, int G, int dk, int dv, int BS, hipStream_t st) {
  const size_t lds = (size_t)(H + G) * dk * sizeof(float);
  static bool attr = false;
  if (lds > 65536 && !attr) {
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&qk_rope_append_kernel<T, V>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, MAX_LDS);
    attr = true;
  }
  hipLaunchKernelGGL((qk_rope_append_kernel<T, V>), dim3(tokens), dim3(256), lds, st, (const T*)qkv, ld, bias, qw, kw, eps, cs,
                     half, vmult, pos, seq_ids, bt, max_blocks, (T*)q, (T*)kc, (T*)vc, H, G, dk, dv, BS);
  DS_CHECK_LAUNCH();
  return 0;
}

}  // namespace

// cs [tokens, half, 2]: cos, sin of pos * freq, times mult
extern "C" int ds_rope_table(const int* pos, const double* freq, float* cs, int tokens, int half, float mult, hipStream_t st) {
  if (tokens <= 0 || half <= 0) return 0;
  const int64_t items = (int64_t)tokens * half;
  hipLaunchKernelGGL(rope_table_kernel, dim3(ds_grid_for(items, 256)), dim3(256), 0, st, pos, freq, (f32x2*)cs, items, half,
                     mult);
  DS_CHECK_LAUNCH();
  return 0;
}

// Rows of qkv `ld` elements apart, [q | k | v]; bias (as long) or null; qw [H dk] and kw [G dk] or null (no norm); cs from
// ds_rope_table with half rotated pairs per head (0: none).
extern "C" int ds_qk_rope_append(const void* qkv, int64_t ld, const float* bias, const float* qw, const float* kw, float eps,
                                 const float* cs, int half, float vmult, const int* pos, const int* seq_ids, const int* bt,
                                 int max_blocks, void* q, void* kc, void* vc, int tokens, int H, int G, int dk, int dv, int BS,
                                 int dtype, hipStream_t st) {
  if (tokens <= 0) return 0;
  if (H <= 0 || G <= 0 || H % G || dk <= 0 || dv <= 0 || BS <= 0 || max_blocks <= 0 || half < 0 || 2 * half > dk ||
      (half && !cs) || ld < (int64_t)(H + G) * dk + (int64_t)G * dv || (int64_t)(H + G) * dk * 4 > MAX_LDS)
    return (int)hipErrorInvalidValue;
  const bool vec = dk % 8 == 0 && dv % 8 == 0 && half % 8 == 0 && ld % 8 == 0 && ((uintptr_t)qkv & 15) == 0 &&
                   (((uintptr_t)bias | (uintptr_t)qw | (uintptr_t)kw) & 15) == 0;
#define GO(T, V)                                                                                                          \
  return launch<T, V>(qkv, ld, bias, qw, kw, eps, cs, half, vmult, pos, seq_ids, bt, max_blocks, q, kc, vc, tokens, H, G, dk, \
                      dv, BS, st)
  if (dtype == DS_F32) {
    if (vec) GO(float, 8);
    GO(float, 1);
  }
  if (dtype == DS_BF16) {
    if (vec) GO(bf16, 8);
    GO(bf16, 1);
  }
#undef GO
  return (int)hipErrorInvalidValue;
}
