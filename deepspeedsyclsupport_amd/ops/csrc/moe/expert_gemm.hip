// Products of mixture-of-experts layers for few rows per expert (decoding, short prompts), any sizes and fp32, CDNA4 (gfx950).
// A pair (token, choice) is entry t * K + k: inputs are read from row entry / div, results written to row `entry`, so nothing
// is copied into expert order and back.
//
//  * stream: bf16 weights streamed once per tile of up to 64 entries. A workgroup owns 32 weight rows of an expert (for the
//    gated form 16 of the gate and the same 16 of the up part, with silu(gate) up as the epilogue); its four waves take
//    alternating 64-wide steps of the inner dimension straight into registers: no LDS, no barrier until the sums meet.
//    Lanes read 32 contiguous bytes per step (the order of the inner dimension is free as long as both operands agree).
//    The entries of an expert come from sorted lists or, for a few hundred of them, are picked out of the routing table by
//    every workgroup itself; then only the experts that occur get workgroups.
//  * any: a workgroup per entry and 64 columns; fp32 and widths that are no multiple of 8.
#include "ds_hip.h"

namespace {

constexpr int MAXE = 256, FEW = 512;

template <int N>
struct Int {
  static constexpr int value = N;
};

__device__ __forceinline__ f32x4 mfma(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ float silu_mul(float g, float u) { return g / (1.f + expf(-g)) * u; }

struct ExpertArgs {
  const void* x;         // [.., K]
  const void* w;         // [E, N, K]; gated: [E, 2 N, K], gate rows first
  void* y;               // [entries, N]
  const int* experts;    // [entries]
  const int* offs;       // [E + 1] and
  const int* order;      // [entries], or null (up to FEW entries)
  int entries, E, N, K, div;
};

// The expert of this workgroup and its entries (list in LDS); their number, 0 for none. block-uniform.
__device__ __forceinline__ int collect(const ExpertArgs& a, int which, int* list, int* words, int& e) {
  const int tid = threadIdx.x, lane = tid & 63;
  if (tid < MAXE / 32) words[tid] = 0;
  __syncthreads();
  for (int i = tid; i < a.entries; i += 256) atomicOr((unsigned*)words + (a.experts[i] >> 5), 1u << (a.experts[i] & 31));
  __syncthreads();
  e = -1;
  int left = which;
#pragma unroll
  for (int i = 0; i < MAXE / 32; ++i) {  // the `which`-th expert that occurs
    unsigned m = words[i];
    const int c = __popc(m);
    if (e < 0 && left < c) {
      for (; left; --left) m &= m - 1;
      e = 32 * i + __ffs(m) - 1;
    }
    if (e < 0) left -= c;
  }
  if (e < 0) return 0;
  if (tid < 64) {  // one wave, in order
    int n = 0;
    for (int b = 0; b < a.entries; b += 64) {
      const bool hit = b + lane < a.entries && a.experts[min(b + lane, a.entries - 1)] == e;
      const unsigned long long m = __ballot(hit);
      if (hit) list[n + __popcll(m & ((1ull << lane) - 1))] = b + lane;
      n += __popcll(m);
    }
    if (lane == 0) words[MAXE / 32] = n;
  }
  __syncthreads();
  return words[MAXE / 32];
}

// MT: tiles of 16 entries at a time
template <int MT, bool GLU>
__global__ void __launch_bounds__(256) expert_stream_kernel(ExpertArgs a) {
  __shared__ int list[FEW], words[MAXE / 32 + 1];
  __shared__ f32x4 red[4][2 * MT][64];
  const int tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, q4 = lane >> 4;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  int e = blockIdx.y, cnt;
  const int* ents = list;
  if (a.offs) {
    cnt = a.offs[e + 1] - a.offs[e];
    ents = a.order + a.offs[e];
  } else {
    cnt = collect(a, blockIdx.y, list, words, e);
  }
  if (cnt == 0) return;
  const int N = a.N, K = a.K, n0 = blockIdx.x * (GLU ? 16 : 32);
  const bf16* w = (const bf16*)a.w + (int64_t)e * (GLU ? 2 : 1) * N * K;
  const bf16* wp[2];
  wp[0] = w + (int64_t)min(n0 + l16, N - 1) * K;
  wp[1] = GLU ? wp[0] + (int64_t)N * K : w + (int64_t)min(n0 + 16 + l16, N - 1) * K;
  for (int m0 = 0; m0 < cnt; m0 += 16 * MT) {
    const bf16* xp[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) xp[m] = (const bf16*)a.x + (int64_t)(ents[min(m0 + 16 * m + l16, cnt - 1)] / a.div) * K;
    f32x4 acc[2][MT];
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int m = 0; m < MT; ++m) acc[i][m] = f32x4{0.f, 0.f, 0.f, 0.f};
    // U steps of the inner dimension: all their loads, then the products
    auto steps = [&](auto count, int k0, bool tail) {
      constexpr int U = decltype(count)::value;
      bf16x8 wv[U][2][2], xv[U][2][MT];
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int c = 0; c < 2; ++c) {
          const int k = k0 + 256 * u + 16 * q4 + 8 * c, kc = tail ? min(k, K - 8) : k;
#pragma unroll
          for (int i = 0; i < 2; ++i) wv[u][c][i] = *reinterpret_cast<const bf16x8*>(wp[i] + kc);
#pragma unroll
          for (int m = 0; m < MT; ++m) xv[u][c][m] = *reinterpret_cast<const bf16x8*>(xp[m] + kc);
          if (tail && k >= K) {  // columns past the width count as zero, on both sides
#pragma unroll
            for (int j = 0; j < 8; ++j) {
#pragma unroll
              for (int i = 0; i < 2; ++i) wv[u][c][i][j] = (bf16)0.f;
#pragma unroll
              for (int m = 0; m < MT; ++m) xv[u][c][m][j] = (bf16)0.f;
            }
          }
        }
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int c = 0; c < 2; ++c)
#pragma unroll
          for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int m = 0; m < MT; ++m) acc[i][m] = mfma(wv[u][c][i], xv[u][c][m], acc[i][m]);
    };
    constexpr int U = MT == 1 ? 4 : 2;
    const int whole = K / 64;
    int s = wid;
    for (; s + 4 * (U - 1) < whole; s += 4 * U) steps(Int<U>{}, 64 * s, false);
    for (; s < whole; s += 4) steps(Int<1>{}, 64 * s, false);
    if (K % 64 && whole % 4 == wid) steps(Int<1>{}, 64 * whole, true);
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int m = 0; m < MT; ++m) red[wid][i * MT + m][lane] = acc[i][m];
    __syncthreads();
    auto total = [&](int j) {
      f32x4 s = red[0][j][lane];
#pragma unroll
      for (int v = 1; v < 4; ++v) s += red[v][j][lane];
      return s;
    };
    // lane: entry l16 of a tile, weight rows 4 q4 .. + 3
    for (int j = wid; j < (GLU ? MT : 2 * MT); j += 4) {
      const int m = j % MT, r = m0 + 16 * m + l16, n = n0 + 4 * q4 + (j / MT) * 16;
      f32x4 v = total(j);
      if constexpr (GLU) {
        const f32x4 u = total(MT + j);
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = silu_mul(v[i], u[i]);
      }
      if (r >= cnt) continue;
      bf16* yr = (bf16*)a.y + (int64_t)ents[r] * N + n;
      if (N % 4 == 0) {
        bf16x4 o;
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] = (bf16)v[i];
        if (n < N) *reinterpret_cast<bf16x4*>(yr) = o;
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (n + i < N) yr[i] = (bf16)v[i];
      }
    }
    __syncthreads();
  }
}

template <typename T, bool GLU>
__global__ void __launch_bounds__(256) expert_any_kernel(ExpertArgs a) {
  const int64_t i = blockIdx.x;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, e = a.experts[i], K = a.K;
  const T* x = (const T*)a.x + i / a.div * K;
  const T* w = (const T*)a.w + (int64_t)e * (GLU ? 2 : 1) * a.N * K;
  for (int n = blockIdx.y * 64 + wid; n < min(a.N, (int)blockIdx.y * 64 + 64); n += 4) {
    const T *wr = w + (int64_t)n * K, *ur = wr + (GLU ? (int64_t)a.N * K : 0);
    float s = 0.f, u = 0.f;
    for (int c = lane; c < K; c += 64) {
      const float xv = (float)x[c];
      s = fmaf(xv, (float)wr[c], s);
      if constexpr (GLU) u = fmaf(xv, (float)ur[c], u);
    }
    s = wave_sum(s);
    if constexpr (GLU) s = silu_mul(s, wave_sum(u));
    if (lane == 0) ((T*)a.y)[i * a.N + n] = (T)s;
  }
}

// out[t] = sum_k w[t, k] y[row(t, k)]
template <typename T>
__global__ void __launch_bounds__(256) expert_sum_kernel(const T* __restrict__ y, const float* __restrict__ w,
                                                         const int* __restrict__ rows, T* __restrict__ out, int W, int K) {
  const int64_t t = blockIdx.x;
  for (int c = threadIdx.x; c < W; c += 256) {
    float v = 0.f;
    for (int k = 0; k < K; ++k) v = fmaf(w[t * K + k], (float)y[(rows ? rows[t * K + k] : t * K + k) * W + c], v);
    out[t * W + c] = (T)v;
  }
}

}  // namespace

extern "C" int ds_expert_few() { return FEW; }

// y[i] = w[experts[i]] x[i / div] for every entry; gated: silu of the first N rows times the others. offs and order from
// ds_expert_place, or null for up to ds_expert_few() entries. `most`: no expert has more entries.
extern "C" int ds_expert_gemm(const void* x, const void* w, void* y, const int* experts, const int* offs, const int* order,
                              int entries, int most, int E, int N, int K, int div, int gated, int dtype, hipStream_t st) {
  if (entries <= 0) return 0;
  if (E <= 0 || E > MAXE || N <= 0 || K <= 0 || div <= 0 || (!offs != !order) || (N + 63) / 64 > 65535)
    return (int)hipErrorInvalidValue;
  const ExpertArgs a{x, w, y, experts, offs, order, entries, E, N, K, div};
  if (dtype == DS_BF16 && K % 8 == 0 && (offs || entries <= FEW)) {
    const dim3 grid((N + (gated ? 15 : 31)) / (gated ? 16 : 32), offs ? E : (entries < E ? entries : E));
#define GO(MT)                                                                                               \
  {                                                                                                          \
    if (gated) hipLaunchKernelGGL((expert_stream_kernel<MT, true>), grid, dim3(256), 0, st, a);              \
    else hipLaunchKernelGGL((expert_stream_kernel<MT, false>), grid, dim3(256), 0, st, a);                   \
  }
    if (most <= 16) GO(1)
    else if (most <= 32) GO(2)
    else GO(4)
#undef GO
    DS_CHECK_LAUNCH();
    return 0;
  }
  const dim3 grid(entries, (N + 63) / 64);
#define GO(T)                                                                                       \
  {                                                                                                 \
    if (gated) hipLaunchKernelGGL((expert_any_kernel<T, true>), grid, dim3(256), 0, st, a);         \
    else hipLaunchKernelGGL((expert_any_kernel<T, false>), grid, dim3(256), 0, st, a);              \
  }
  if (dtype == DS_F32) GO(float)
  else if (dtype == DS_BF16) GO(bf16)
  else return (int)hipErrorInvalidValue;
#undef GO
  DS_CHECK_LAUNCH();
  return 0;
}

extern "C" int ds_expert_sum(const void* y, const float* w, const int* rows, void* out, int T, int W, int K, int dtype,
                             hipStream_t st) {
  if (T <= 0) return 0;
  if (W <= 0 || K <= 0) return (int)hipErrorInvalidValue;
  if (dtype == DS_F32)
    hipLaunchKernelGGL(expert_sum_kernel<float>, dim3(T), dim3(256), 0, st, (const float*)y, w, rows, (float*)out, W, K);
  else if (dtype == DS_BF16)
    hipLaunchKernelGGL(expert_sum_kernel<bf16>, dim3(T), dim3(256), 0, st, (const bf16*)y, w, rows, (bf16*)out, W, K);
  else return (int)hipErrorInvalidValue;
  DS_CHECK_LAUNCH();
  return 0;
}
