// Exponential input and forget gates with a running maximum (matrix memories whose gates are kept as logarithms), CDNA4
// (gfx950).
//
// Per head, from projected columns x_i and x_f:  i = cap tanh((x_i + b_i) / cap),  f = logsigmoid(cap tanh((x_f + b_f) / cap)),
//     m_t = max(f_t + m_(t-1), i_t),   m_(-1) = 0
// and the recurrence relative to e^m is S <- e^{f + m_(t-1) - m_t} S + e^{i - m_t} k v^T: a scan with a decay and a step size per
// token, which is what decayed_scan.hip and decayed_chunk.hip run. The read-out's floor is e^{-m_t}.
//
// t -> m_t is a composition of maps m -> max(F + m, I), so a workgroup per (sequence, head) takes as many tokens at once as
// it has threads: shuffles within a wave, LDS between the waves. Any rounding of m cancels: it only names the scale that state
// and gates are kept in.
#include "ds_hip.h"

namespace {

struct MaxPlus {  // m -> max(F + m, I)
  float F, I;
};
__device__ __forceinline__ MaxPlus then(MaxPlus a, MaxPlus b) { return {a.F + b.F, fmaxf(b.F + a.I, b.I)}; }

template <typename T, int NT>
__global__ void __launch_bounds__(NT) exp_gates_kernel(const T* __restrict__ proj, int rows, int ci, int cf,
                                                       const float* __restrict__ bi, const float* __restrict__ bf, float cap,
                                                       float* __restrict__ peak, const int* __restrict__ cu,
                                                       const int* __restrict__ start, const int* __restrict__ slots,
                                                       float* __restrict__ gb, float* __restrict__ floors, int H) {
  constexpr int NW = NT / 64;
  __shared__ MaxPlus tot[NW];
  __shared__ float last;
  const int seq = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int t0 = cu[seq], n = cu[seq + 1] - t0;
  float* mp = peak + (int64_t)slots[seq] * H + h;
  float m = start[seq] == 0 ? 0.f : *mp;
  const float b_i = bi[h], b_f = bf[h];
  for (int base = 0; base < n; base += NT) {  // (uniform over the workgroup)
    const int t = base + tid;
    const bool ok = t < n;
    float i = -INFINITY, f = 0.f;
    if (ok) {
      const T* row = proj + (int64_t)(t0 + t) * rows;
      i = cap * tanhf(((float)row[ci + h] + b_i) / cap);
      const float z = cap * tanhf(((float)row[cf + h] + b_f) / cap);
      f = fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
    }
    MaxPlus s{f, i};
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const MaxPlus p{__shfl_up(s.F, o, 64), __shfl_up(s.I, o, 64)};
      if (lane >= o) s = then(p, s);
    }
    float mw = m;  // the maximum before this wave's first token
    if constexpr (NW > 1) {
      if (lane == 63) tot[w] = s;
      __syncthreads();
      for (int k = 0; k < w; ++k) mw = fmaxf(tot[k].F + mw, tot[k].I);
    }
    const float mt = fmaxf(s.F + mw, s.I);
    float mprev = __shfl_up(mt, 1, 64);
    if (lane == 0) mprev = mw;
    if (ok) {
      const int64_t tok = t0 + t;
      gb[tok * 2 * H + h] = f + mprev - mt;
      gb[(tok * 2 + 1) * H + h] = expf(i - mt);
      floors[tok * H + h] = expf(-mt);
    }
    if (tid == NT - 1) last = mt;  // (threads past the end hand the maximum on)
    __syncthreads();
    m = last;
    __syncthreads();
  }
  if (tid == 0 && n > 0) *mp = m;
}

}  // namespace

// Columns ci .. ci + H and cf .. cf + H of proj [tokens, rows]; peak [slots, H] advances. -> gb [tokens, 2, H] (log decay, step
// size), floors [tokens, H]. `longest`: tokens of the longest portion.
extern "C" int ds_exp_gates(const void* proj, int rows, int ci, int cf, const float* bi, const float* bf, float cap,
                            float* peak, const int* cu, const int* start, const int* slots, float* gb, float* floors, int nseq,
                            int longest, int H, int dtype, hipStream_t st) {
  if (nseq <= 0) return 0;
  if (H <= 0 || H > 65535 || ci < 0 || cf < 0 || ci + H > rows || cf + H > rows || !(cap > 0.f)) return (int)hipErrorInvalidValue;
#define GO(T, NT)                                                                                                    \
  hipLaunchKernelGGL((exp_gates_kernel<T, NT>), dim3(nseq, H), dim3(NT), 0, st, (const T*)proj, rows, ci, cf, bi, bf, cap, \
                     peak, cu, start, slots, gb, floors, H)
  if (dtype == DS_F32) {
    if (longest <= 64) GO(float, 64);
    else GO(float, 1024);
  } else if (dtype == DS_BF16) {
    if (longest <= 64) GO(bf16, 64);
    else GO(bf16, 1024);
  } else {
    return (int)hipErrorInvalidValue;
  }
#undef GO
  DS_CHECK_LAUNCH();
  return 0;
}
