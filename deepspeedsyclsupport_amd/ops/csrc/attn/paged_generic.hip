// Ragged paged attention for any head sizes in fp32 or bf16, CDNA4 (gfx950): the path of 32-bit models and of head
// sizes the MFMA kernels (paged_prefill.hip, decode_attn.hip) do not tile. Prefill rows and decode rows alike.
//
// One wave per (token, query head): 64 keys at a time, a lane per key for the scores, then a lane per value column
// for the weighted sum. Scores, softmax and sums are fp32. A key j is visible to position i if lo(i) <= j <= i, where
// lo is i - window + 1 (sliding window), the start of i's chunk (chunked attention), or 0. Optional tanh soft cap;
// optional sink: exp(sink of the head) joins the softmax's denominator; optional gate: the head's output times the sigmoid of a
// number per token and head. Value rows may lie further apart than their
// width: latent attention's values are the first columns of its keys.
#include "ds_hip.h"

namespace {

constexpr int MAXD = 1024;  // query / key width (LDS) and value width (16 columns per lane)

template <typename T>
__global__ void __launch_bounds__(64) paged_generic_kernel(
    const T* __restrict__ q, const T* __restrict__ kc, const T* __restrict__ vc, T* __restrict__ o,
    const int* __restrict__ block_table, int max_blocks, const int* __restrict__ pos, const int* __restrict__ seq_ids,
    int H, int G, int dk, int dv, int vrow, int BS, float scale, float softcap, int window, int chunk,
    const float* __restrict__ sink, int64_t ldo, const T* __restrict__ gate, int64_t ldg) {
  __shared__ float qs[MAXD];
  __shared__ float ps[64];
  __shared__ int64_t slot_s[64];
  const int t = blockIdx.x, h = blockIdx.y, g = h / (H / G), lane = threadIdx.x;
  const int p = pos[t];
  const int* bt = block_table + (int64_t)seq_ids[t] * max_blocks;
  const T* qr = q + ((int64_t)t * H + h) * dk;
  for (int c = lane; c < dk; c += 64) qs[c] = (float)qr[c];
  __syncthreads();
  int lo = 0;
  if (chunk > 0) lo = p / chunk * chunk;
  if (window > 0) lo = max(lo, p - window + 1);
  float m = -INFINITY, l = 0.f, acc[MAXD / 64];
#pragma unroll
  for (int i = 0; i < MAXD / 64; ++i) acc[i] = 0.f;
  for (int k0 = lo; k0 <= p; k0 += 64) {
    const int key = k0 + lane, kk = min(key, p);
    const int64_t slot = ((int64_t)bt[kk / BS] * G + g) * BS + kk % BS;
    const T* kr = kc + slot * dk;
    float s = 0.f;
    for (int c = 0; c < dk; ++c) s = fmaf(qs[c], (float)kr[c], s);
    s *= scale;
    if (softcap > 0.f) s = softcap * tanhf(s / softcap);
    if (key > p) s = -INFINITY;
    const float mn = fmaxf(m, wave_max(s));  // finite: the first key of every tile is visible
    const float w = expf(s - mn), alpha = expf(m - mn);
    l = l * alpha + wave_sum(w);
    m = mn;
    ps[lane] = w;
    slot_s[lane] = slot;
    __syncthreads();
    const int nk = min(64, p - k0 + 1);
#pragma unroll
    for (int i = 0; i < MAXD / 64; ++i) {
      const int c = i * 64 + lane;
      if (i * 64 >= dv) break;
      float a = acc[i] * alpha;
      if (c < dv)
        for (int j = 0; j < nk; ++j) a = fmaf(ps[j], (float)vc[slot_s[j] * vrow + c], a);
      acc[i] = a;
    }
    __syncthreads();
  }
  if (sink) {  // (in the frame of the maximum; a sink far above every score takes all the weight)
    const float mn = fmaxf(m, sink[h]), alpha = expf(m - mn);
    l = l * alpha + expf(sink[h] - mn);
#pragma unroll
    for (int i = 0; i < MAXD / 64; ++i) acc[i] *= alpha;
  }
  if (gate) l *= 1.f + expf(-(float)gate[t * ldg + h]);
  T* orow = o + t * ldo + h * dv;
#pragma unroll
  for (int i = 0; i < MAXD / 64; ++i) {
    const int c = i * 64 + lane;
    if (c < dv) orow[c] = (T)(acc[i] / l);
  }
}

}  // namespace

extern "C" int ds_paged_generic(const void* q, const void* kc, const void* vc, void* o, const int* bt, int max_blocks,
                                const int* pos, const int* seq_ids, int tokens, int H, int G, int dk, int dv, int vrow,
                                int BS, float scale, float softcap, int window, int chunk, const float* sink, int64_t ldo,
                                const void* gate, int64_t ldg, int dtype, hipStream_t st) {
  if (tokens <= 0) return 0;
  if (G <= 0 || H % G || dk <= 0 || dv <= 0 || vrow < dv || dk > MAXD || dv > MAXD || BS <= 0 || H > 65535 ||
      ldo < (int64_t)H * dv)
    return (int)hipErrorInvalidValue;
#define GO(T)                                                                                                        \
  hipLaunchKernelGGL((paged_generic_kernel<T>), dim3(tokens, H), dim3(64), 0, st, (const T*)q, (const T*)kc,         \
                     (const T*)vc, (T*)o, bt, max_blocks, pos, seq_ids, H, G, dk, dv, vrow, BS, scale, softcap, window, chunk, \
                     sink, ldo, (const T*)gate, ldg)
  if (dtype == DS_F32) GO(float);
  else if (dtype == DS_BF16) GO(bf16);
  else return (int)hipErrorInvalidValue;
#undef GO
  DS_CHECK_LAUNCH();
  return 0;
}
