// Routing of mixture-of-experts layers with grouped experts, CDNA4 (gfx950).
//
//  * route: router logits in fp32 (bf16 operands through the matrix cores, or plain fp32 products), scores (the softmax over all
//    experts, or every expert's sigmoid), the best groups of neighbouring experts (a group is as good as its best member, or its
//    two best together), the best experts within those, weights divided by their sum, times a constant. One launch: the logits
//    of a tile of tokens never leave LDS. Ties go to the lower index.
//  * place: the (token, choice) pairs sorted by expert, as lists for the expert products (expert_gemm.hip). The counts come
//    from the routing kernel; nothing waits for the host.
#include "ds_hip.h"

namespace {

constexpr int MAXE = 256, MAXK = 64;

template <int N>
struct Int {
  static constexpr int value = N;
};

__device__ __forceinline__ f32x4 mfma(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

struct RouteArgs {
  int T, W, E, K, groups, keep, sigmoid, best;   // best: members that count for a group, 1 or 2
  float scale;
  int* experts;      // [T, K]
  float* weights;    // [T, K]
  int* counts;       // [E], zero before; null: no lists wanted
  int* slots;        // [T, K]: place of the pair within its expert's
};

// One wave: logits z [E] of a token in LDS (overwritten), gs scratch [groups]
__device__ __forceinline__ void choose(float* z, float* gs, int tok, const RouteArgs& a, int* hist) {
  const int lane = threadIdx.x & 63, E = a.E, per = E / a.groups;
  float s[MAXE / 64], mx = -INFINITY, den = 0.f;
#pragma unroll
  for (int i = 0; i < MAXE / 64; ++i) {
    s[i] = lane + 64 * i < E ? z[lane + 64 * i] : -INFINITY;
    mx = fmaxf(mx, s[i]);
  }
  if (a.sigmoid) {
#pragma unroll
    for (int i = 0; i < MAXE / 64; ++i) s[i] = 1.f / (1.f + expf(-s[i]));
  } else {
    mx = wave_max(mx);
#pragma unroll
    for (int i = 0; i < MAXE / 64; ++i) {
      s[i] = lane + 64 * i < E ? expf(s[i] - mx) : 0.f;
      den += s[i];
    }
    den = wave_sum(den);
#pragma unroll
    for (int i = 0; i < MAXE / 64; ++i) s[i] /= den;
  }
#pragma unroll
  for (int i = 0; i < MAXE / 64; ++i)
    if (lane + 64 * i < E) z[lane + 64 * i] = s[i];
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  for (int g = lane; g < a.groups; g += 64) {
    float b = 0.f, c = 0.f;
    for (int e = g * per; e < (g + 1) * per; ++e) {
      c = fmaxf(c, fminf(b, z[e]));
      b = fmaxf(b, z[e]);
    }
    gs[g] = a.best == 2 ? b + c : b;
  }
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
#pragma unroll
  for (int i = 0; i < MAXE / 64; ++i) {
    const int e = lane + 64 * i;
    if (e >= E) {
      s[i] = -1.f;
      continue;
    }
    const int g = e / per;
    const float b = gs[g];
    int better = 0;
    for (int o = 0; o < a.groups; ++o) better += gs[o] > b || (gs[o] == b && o < g);
    if (better >= a.keep) s[i] = -1.f;
  }
  float mine = 0.f, sum = 0.f;  // lane k keeps choice k
  int my_e = 0;
  for (int k = 0; k < a.K; ++k) {
    float bv = -1.f;
    int be = MAXE;
#pragma unroll
    for (int i = 0; i < MAXE / 64; ++i)
      if (s[i] > bv) {
        bv = s[i];
        be = lane + 64 * i;
      }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(bv, o, 64);
      const int oe = __shfl_xor(be, o, 64);
      if (ov > bv || (ov == bv && oe < be)) {
        bv = ov;
        be = oe;
      }
    }
#pragma unroll
    for (int i = 0; i < MAXE / 64; ++i)
      if (be == lane + 64 * i) s[i] = -1.f;
    be = min(be, E - 1);      // (logits that are not numbers choose nothing: stay in bounds)
    sum += bv;
    if (lane == k) {
      mine = bv;
      my_e = be;
    }
  }
  if (lane < a.K) {
    const int64_t i = (int64_t)tok * a.K + lane;
    a.experts[i] = my_e;
    a.weights[i] = mine / (sum + 1e-20f) * a.scale;
    if (hist) a.slots[i] = atomicAdd(hist + my_e, 1);  // within the workgroup; the base is added below
  }
}

// The workgroup's pairs take a run of every expert's places
__device__ __forceinline__ void claim(const RouteArgs& a, int first, int n, int* hist) {
  __syncthreads();
  for (int e = threadIdx.x; e < a.E; e += blockDim.x)
    if (const int c = hist[e]) hist[e] = atomicAdd(a.counts + e, c);
  __syncthreads();
  for (int i = threadIdx.x; i < n * a.K; i += blockDim.x) {
    const int64_t p = (int64_t)first * a.K + i;
    a.slots[p] += hist[a.experts[p]];
  }
}

// bf16, W a multiple of 8. NW waves share the width of 16 TM tokens and up to 16 ET experts.
template <int ET, int TM, int NW>
__global__ void __launch_bounds__(64 * NW) route_mfma_kernel(const bf16* __restrict__ h, const bf16* __restrict__ rw,
                                                             RouteArgs a) {
  constexpr int TOK = 16 * TM, ZP = 16 * ET + 1;
  __shared__ float z[TOK * ZP];
  __shared__ f32x4 red[NW / 2][TM * ET][64];
  __shared__ float gs[NW][16 * ET];
  __shared__ int hist[MAXE];
  const int tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, q4 = lane >> 4, w = tid >> 6;
  const int t0 = blockIdx.x * TOK, n = min(TOK, a.T - t0);
  for (int e = tid; e < MAXE; e += 64 * NW) hist[e] = 0;
  f32x4 acc[TM][ET];
#pragma unroll
  for (int m = 0; m < TM; ++m)
#pragma unroll
    for (int e = 0; e < ET; ++e) acc[m][e] = f32x4{0.f, 0.f, 0.f, 0.f};
  const bf16 *hp[TM], *wp[ET];
#pragma unroll
  for (int m = 0; m < TM; ++m) hp[m] = h + (int64_t)(t0 + min(16 * m + l16, n - 1)) * a.W;
#pragma unroll
  for (int e = 0; e < ET; ++e) wp[e] = rw + (int64_t)min(16 * e + l16, a.E - 1) * a.W;
  // U steps of 32 of the width: all their loads, then the products
  auto steps = [&](auto count, int k0, bool tail) {
    constexpr int U = decltype(count)::value;
    bf16x8 x[U][TM], y[U][ET];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + 32 * NW * u + 8 * q4, kc = tail ? min(k, a.W - 8) : k;
#pragma unroll
      for (int e = 0; e < ET; ++e) y[u][e] = *reinterpret_cast<const bf16x8*>(wp[e] + kc);
#pragma unroll
      for (int m = 0; m < TM; ++m) x[u][m] = *reinterpret_cast<const bf16x8*>(hp[m] + kc);
      if (tail && k >= a.W) {  // the last step may reach past the width
#pragma unroll
        for (int m = 0; m < TM; ++m)
#pragma unroll
          for (int j = 0; j < 8; ++j) x[u][m][j] = (bf16)0.f;
      }
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int m = 0; m < TM; ++m)
#pragma unroll
        for (int e = 0; e < ET; ++e) acc[m][e] = mfma(y[u][e], x[u][m], acc[m][e]);
  };
  constexpr int U = ET <= 2 ? 8 : ET <= 4 ? 4 : 2;
  const int whole = a.W / 32;
  int k = w;
  for (; k + NW * (U - 1) < whole; k += NW * U) steps(Int<U>{}, 32 * k, false);
  for (; k < whole; k += NW) steps(Int<1>{}, 32 * k, false);
  if (a.W % 32 && whole % NW == w) steps(Int<1>{}, 32 * whole, true);
#pragma unroll
  for (int half = NW / 2; half >= 1; half /= 2) {  // the waves' shares, pairwise
    if (w >= half && w < 2 * half) {
#pragma unroll
      for (int m = 0; m < TM; ++m)
#pragma unroll
        for (int e = 0; e < ET; ++e) red[w - half][m * ET + e][lane] = acc[m][e];
    }
    __syncthreads();
    if (w < half) {
#pragma unroll
      for (int m = 0; m < TM; ++m)
#pragma unroll
        for (int e = 0; e < ET; ++e) acc[m][e] += red[w][m * ET + e][lane];
    }
    __syncthreads();
  }
  if (w == 0) {
#pragma unroll
    for (int m = 0; m < TM; ++m)
#pragma unroll
      for (int e = 0; e < ET; ++e)
#pragma unroll
        for (int r = 0; r < 4; ++r)  // token 16 m + l16, expert 16 e + 4 q4 + r
          z[(16 * m + l16) * ZP + 16 * e + 4 * q4 + r] = acc[m][e][r];
  }
  __syncthreads();
  for (int i = w; i < n; i += NW) choose(z + i * ZP, gs[w], t0 + i, a, a.counts ? hist : nullptr);
  if (a.counts) claim(a, t0, n, hist);
}

// fp32, or widths the matrix kernel does not take: a workgroup per token
template <typename T>
__global__ void __launch_bounds__(256) route_any_kernel(const T* __restrict__ h, const T* __restrict__ rw, RouteArgs a) {
  __shared__ float z[MAXE], gs[MAXE];
  __shared__ int hist[MAXE];
  const int t = blockIdx.x, lane = threadIdx.x & 63;
  const T* x = h + (int64_t)t * a.W;
  for (int e = threadIdx.x; e < MAXE; e += 256) hist[e] = 0;
  for (int e = threadIdx.x >> 6; e < a.E; e += 4) {
    const T* y = rw + (int64_t)e * a.W;
    float s = 0.f;
    for (int c = lane; c < a.W; c += 64) s = fmaf((float)x[c], (float)y[c], s);
    s = wave_sum(s);
    if (lane == 0) z[e] = s;
  }
  __syncthreads();
  if (threadIdx.x < 64) choose(z, gs, t, a, a.counts ? hist : nullptr);
  if (a.counts) claim(a, t, 1, hist);
}

// Exclusive prefix of counts [E] in LDS (pre[E]: the total), by the first wave
__device__ __forceinline__ void prefix(const int* counts, int E, int* pre) {
  if (threadIdx.x < 64) {
    const int lane = threadIdx.x;
    int c[4], s = 0;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      c[i] = 4 * lane + i < E ? counts[4 * lane + i] : 0;
      s += c[i];
    }
    int run = s;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int y = __shfl_up(run, o, 64);
      if (lane >= o) run += y;
    }
    int at = run - s;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (4 * lane + i < E) pre[4 * lane + i] = at;
      at += c[i];
    }
    if (lane == 63) pre[E] = run;
  }
  __syncthreads();
}

__global__ void __launch_bounds__(256) place_kernel(const int* __restrict__ experts, const int* __restrict__ slots,
                                                    const int* __restrict__ counts, int* __restrict__ offs,
                                                    int* __restrict__ order, int* __restrict__ rows, int entries, int E) {
  __shared__ int pre[MAXE + 1];
  prefix(counts, E, pre);
  if (blockIdx.x == 0)
    for (int e = threadIdx.x; e <= E; e += 256) offs[e] = pre[e];
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= entries) return;
  const int r = pre[experts[i]] + slots[i];
  order[r] = i;
  rows[i] = r;
}

// xs[rows[t, k]] = x[t]: a workgroup per token
__global__ void __launch_bounds__(256) spread_kernel(const f32x4* __restrict__ x, const int* __restrict__ rows,
                                                     f32x4* __restrict__ xs, int W16, int K) {
  const int64_t t = blockIdx.x;
  for (int c = threadIdx.x; c < W16; c += 256) {
    const f32x4 v = x[t * W16 + c];
    for (int k = 0; k < K; ++k) xs[(int64_t)rows[t * K + k] * W16 + c] = v;
  }
}

}  // namespace

// h [T, W], router [E, W] -> experts, weights [T, K]; with counts (zero) and slots also the places of all pairs
extern "C" int ds_route(const void* h, const void* router, int* experts, float* weights, int* counts, int* slots, int T, int W,
                        int E, int K, int groups, int keep, int sigmoid, int best, float scale, int dtype, hipStream_t st) {
  if (T <= 0) return 0;
  if (W <= 0 || E <= 0 || E > MAXE || K <= 0 || K > MAXK || groups <= 0 || E % groups || keep <= 0 || keep > groups ||
      K > keep * (E / groups) || (!counts != !slots) || best < 1 || best > 2)
    return (int)hipErrorInvalidValue;
  const RouteArgs a{T, W, E, K, groups, keep, sigmoid, best, scale, experts, weights, counts, slots};
  if (dtype == DS_BF16 && W % 8 == 0) {
#define GO(ET, TM, NW)                                                                                              \
  hipLaunchKernelGGL((route_mfma_kernel<ET, TM, NW>), dim3((T + 16 * TM - 1) / (16 * TM)), dim3(64 * NW), 0, st,     \
                     (const bf16*)h, (const bf16*)router, a)
    const bool wide = T > 4096;
    if (E <= 16) {
      if (wide) GO(1, 2, 8);
      else GO(1, 1, 16);
    } else if (E <= 32) {
      if (wide) GO(2, 2, 8);
      else GO(2, 1, 16);
    } else if (E <= 64) {
      if (wide) GO(4, 2, 8);
      else GO(4, 1, 8);
    } else if (E <= 128) GO(8, 1, 8);
    else GO(16, 1, 4);
#undef GO
  } else if (dtype == DS_BF16) {
    hipLaunchKernelGGL(route_any_kernel<bf16>, dim3(T), dim3(256), 0, st, (const bf16*)h, (const bf16*)router, a);
  } else if (dtype == DS_F32) {
    hipLaunchKernelGGL(route_any_kernel<float>, dim3(T), dim3(256), 0, st, (const float*)h, (const float*)router, a);
  } else {
    return (int)hipErrorInvalidValue;
  }
  DS_CHECK_LAUNCH();
  return 0;
}

// -> offs [E + 1], order [entries] (pairs by expert), rows [entries] (a pair's place in it)
extern "C" int ds_expert_place(const int* experts, const int* slots, const int* counts, int* offs, int* order, int* rows,
                               int entries, int E, hipStream_t st) {
  if (entries <= 0) return 0;
  if (E <= 0 || E > MAXE) return (int)hipErrorInvalidValue;
  hipLaunchKernelGGL(place_kernel, dim3((entries + 255) / 256), dim3(256), 0, st, experts, slots, counts, offs, order, rows,
                     entries, E);
  DS_CHECK_LAUNCH();
  return 0;
}

// row_bytes: of a row, a multiple of 16
extern "C" int ds_expert_spread(const void* x, const int* rows, void* xs, int T, int K, int64_t row_bytes, hipStream_t st) {
  if (T <= 0) return 0;
  if (K <= 0 || row_bytes <= 0 || row_bytes % 16) return (int)hipErrorInvalidValue;
  hipLaunchKernelGGL(spread_kernel, dim3(T), dim3(256), 0, st, (const f32x4*)x, rows, (f32x4*)xs, (int)(row_bytes / 16), K);
  DS_CHECK_LAUNCH();
  return 0;
}
