// QKV epilogue of attention layers with per-head query / key RMSNorm, CDNA4 (gfx950).
//
// One wave per (token, head) of rows that may be columns of wider ones: q and k heads are optionally rotated (pairs of
// neighbours, by a table of cosines and sines per token), divided by their root mean square and optionally scaled by a shared
// weight; v heads are optionally mixed with the values of an earlier layer (v <- (1 - lambda) v + lambda v_first); q is written
// out, k and v go straight into the paged cache, whose key and value rows may differ in width.
#include "ds_hip.h"

namespace {

struct Turn {
  const float* cs;  // [tokens, half, 2] or null
  int half;         // rotated pairs (2 i, 2 i + 1) of a head
};

template <typename T>
__global__ void __launch_bounds__(256) qk_norm_append_kernel(
    const T* __restrict__ qkv, const float* __restrict__ qw, const float* __restrict__ kw, float eps,
    const T* __restrict__ vfirst, int64_t vf_stride, const float* __restrict__ lambda, const int* __restrict__ pos,
    const int* __restrict__ seq_ids, const int* __restrict__ block_table, int max_blocks, T* __restrict__ q_out,
    T* __restrict__ kc, T* __restrict__ vc, int tokens, int H, int G, int dk, int dv, int BS, int64_t ld, Turn turn) {
  const int slots = H + 2 * G, lane = threadIdx.x & 63;
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= (int64_t)tokens * slots) return;
  const int t = (int)(item / slots), h = (int)(item % slots);
  const T* row = qkv + t * ld;
  int64_t slot = 0;
  if (h >= H) {
    const int p = pos[t];
    const int g = h < H + G ? h - H : h - H - G;
    slot = ((int64_t)block_table[(int64_t)seq_ids[t] * max_blocks + p / BS] * G + g) * BS + p % BS;
  }
  if (h >= H + G) {
    const int g = h - H - G;
    const T* v = row + (int64_t)(H + G) * dk + (int64_t)g * dv;
    const float lam = vfirst ? lambda[0] : 0.f;
    for (int c = lane; c < dv; c += 64) {
      float a = (float)v[c];
      if (vfirst) a = (1.f - lam) * a + lam * (float)vfirst[(int64_t)t * vf_stride + (int64_t)g * dv + c];
      vc[slot * dv + c] = (T)a;
    }
    return;
  }
  const T* src = row + (int64_t)h * dk;
  const float* cs = turn.cs + (int64_t)t * turn.half * 2;
  auto column = [&](int c) {
    const float a = (float)src[c];
    if (c >= 2 * turn.half) return a;
    const float b = (float)src[c ^ 1], co = cs[c & ~1], si = cs[c | 1];
    return c & 1 ? a * co + b * si : a * co - b * si;
  };
  float ss = 0.f;
  for (int c = lane; c < dk; c += 64) {
    const float a = column(c);
    ss = fmaf(a, a, ss);
  }
  const float rs = 1.f / sqrtf(wave_sum(ss) / (float)dk + eps);
  T* dst = h < H ? q_out + ((int64_t)t * H + h) * dk : kc + slot * dk;
  const float* w = h < H ? qw : kw;
  for (int c = lane; c < dk; c += 64) dst[c] = (T)(column(c) * (w ? rs * w[c] : rs));
}

// The same for head widths that are multiples of 8: LPH lanes per head with 8 elements each, 64 / LPH heads per wave
template <typename T, int LPH>
__global__ void __launch_bounds__(256) qk_norm_append_vec_kernel(
    const T* __restrict__ qkv, const float* __restrict__ qw, const float* __restrict__ kw, float eps,
    const T* __restrict__ vfirst, int64_t vf_stride, const float* __restrict__ lambda, const int* __restrict__ pos,
    const int* __restrict__ seq_ids, const int* __restrict__ block_table, int max_blocks, T* __restrict__ q_out,
    T* __restrict__ kc, T* __restrict__ vc, int tokens, int H, int G, int dk, int dv, int BS, int64_t ld, Turn turn) {
  constexpr int HPB = 256 / LPH;
  const int slots = H + 2 * G, li = threadIdx.x % LPH, c = li * 8;
  const int64_t item = (int64_t)blockIdx.x * HPB + threadIdx.x / LPH;
  if (item >= (int64_t)tokens * slots) return;  // whole lane groups
  const int t = (int)(item / slots), h = (int)(item % slots);
  const T* row = qkv + t * ld;
  const bool is_v = h >= H + G;
  const int width = is_v ? dv : dk;
  const T* src = row + (is_v ? (int64_t)(H + G) * dk + (int64_t)(h - H - G) * dv : (int64_t)h * dk);
  int64_t slot = 0;
  if (h >= H) {
    const int p = pos[t], g = is_v ? h - H - G : h - H;
    slot = ((int64_t)block_table[(int64_t)seq_ids[t] * max_blocks + p / BS] * G + g) * BS + p % BS;
  }
  const bool on = c < width;
  float x[8];
  Vec8<T>::load(src + (on ? c : 0), x);
  if (is_v) {
    if (vfirst) {
      const float lam = lambda[0];
      const T* vf = vfirst + (int64_t)t * vf_stride + (int64_t)(h - H - G) * dv + (on ? c : 0);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[j] = (1.f - lam) * x[j] + lam * (float)vf[j];
    }
    if (on) Vec8<T>::store(vc + slot * dv + c, x);
    return;
  }
  if (c < 2 * turn.half) {
    const float* cs = turn.cs + (int64_t)t * turn.half * 2 + c;
#pragma unroll
    for (int j = 0; j < 8; j += 2) {
      if (c + j >= 2 * turn.half) break;
      const float u = x[j], v = x[j + 1], co = cs[j], si = cs[j + 1];
      x[j] = u * co - v * si;
      x[j + 1] = v * co + u * si;
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < 8; ++j) ss = fmaf(x[j], x[j], ss);
  if (!on) ss = 0.f;
#pragma unroll
  for (int o = LPH / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
  const float rs = 1.f / sqrtf(ss / (float)dk + eps);
  if (!on) return;
  const float* wp = h < H ? qw : kw;
  if (wp) {
    float w[8];
    Vec8<float>::load(wp + c, w);
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] *= rs * w[j];
  } else {
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] *= rs;
  }
  Vec8<T>::store((h < H ? q_out + ((int64_t)t * H + h) * dk : kc + slot * dk) + c, x);
}

template <typename T>
int launch(const void* qkv, const float* qw, const float* kw, float eps, const void* vfirst, int64_t vf_stride,
           const float* lambda, const int* pos, const int* seq_ids, const int* bt, int max_blocks, void* q, void* kc,
           void* vc, int tokens, int H, int G, int dk, int dv, int BS, int64_t ld, const Turn& turn, hipStream_t st) {
  const int64_t items = (int64_t)tokens * (H + 2 * G);
  if (dk % 8 == 0 && dv % 8 == 0 && dk <= 256 && dv <= 256 && ld % 8 == 0 && ((uintptr_t)qkv & 15) == 0) {
#define VEC(LPH)                                                                                                    \
  hipLaunchKernelGGL((qk_norm_append_vec_kernel<T, LPH>), dim3((unsigned)((items * LPH + 255) / 256)), dim3(256), 0, st, \
                     (const T*)qkv, qw, kw, eps, (const T*)vfirst, vf_stride, lambda, pos, seq_ids, bt, max_blocks, (T*)q, \
                     (T*)kc, (T*)vc, tokens, H, G, dk, dv, BS, ld, turn)
    if (dk <= 64 && dv <= 64) VEC(8);
    else if (dk <= 128 && dv <= 128) VEC(16);
    else VEC(32);
#undef VEC
    DS_CHECK_LAUNCH();
    return 0;
  }
  hipLaunchKernelGGL((qk_norm_append_kernel<T>), dim3((unsigned)((items + 3) / 4)), dim3(256), 0, st, (const T*)qkv, qw,
                     kw, eps, (const T*)vfirst, vf_stride, lambda, pos, seq_ids, bt, max_blocks, (T*)q, (T*)kc, (T*)vc,
                     tokens, H, G, dk, dv, BS, ld, turn);
  DS_CHECK_LAUNCH();
  return 0;
}

}  // namespace

// Rows of qkv `ld` elements apart, [q | k | v]; qw, kw [dk] or null; cs [tokens, half, 2] or null
extern "C" int ds_qk_norm_append(const void* qkv, int64_t ld, const float* cs, int half, const float* qw, const float* kw, float eps, const void* vfirst,
                                 int64_t vf_stride, const float* lambda, const int* pos, const int* seq_ids,
                                 const int* bt, int max_blocks, void* q, void* kc, void* vc, int tokens, int H, int G,
                                 int dk, int dv, int BS, int dtype, hipStream_t st) {
  if (tokens <= 0) return 0;
  if (H <= 0 || G <= 0 || H % G || dk <= 0 || dv <= 0 || BS <= 0 || max_blocks <= 0 || (vfirst && !lambda) ||
      ld < (int64_t)(H + G) * dk + (int64_t)G * dv || half < 0 || 2 * half > dk || (half && !cs))
    return (int)hipErrorInvalidValue;
#define GO(T) \
  launch<T>(qkv, qw, kw, eps, vfirst, vf_stride, lambda, pos, seq_ids, bt, max_blocks, q, kc, vc, tokens, H, G, dk, dv, BS, ld, \
            Turn{cs, half}, st)
  if (dtype == DS_F32) return GO(float);
  if (dtype == DS_BF16) return GO(bf16);
#undef GO
  return (int)hipErrorInvalidValue;
}
