// Selective scan: recurrences with a decay of their own per channel and state, CDNA4 (gfx950).
//
// Every channel c carries N numbers in fp32 that start at zero. With step = softplus(dt + dt_bias) and A = -exp(A_log):
//     S[c, n] <- exp(step_c A[c, n]) S[c, n] + step_c x_c B_n;   y_c = sum_n S[c, n] C_n + D_c x_c;   out_c = y_c silu(z_c)
// B and C belong to the token, shared by all channels. One exponential and four multiplications per number and token: bound by
// the vector unit (the exponential takes a quarter of its rate), so there is nothing for the matrix cores to do.
//
// A workgroup of four waves takes 256 / LP neighbouring channels of one sequence and walks its new tokens, TT at a time. LP lanes
// share a channel, NPL numbers each, in registers throughout. LP is chosen so that the waves cover the chip: few lanes per
// channel spend the least on what a channel does once per token, many make a single long sequence parallel.
//  * stage: step and step * x of every (token, channel) of the tile, B and C, all fp32, into LDS; x and z stay with the thread
//    that will write the same (token, channel). The next tile's operands are on their way meanwhile.
//  * walk: token by token without barriers. Partial sums of y meet across the LP lanes; lane i keeps those of token i of LP.
//  * write: y from LDS, skip and gate applied, in whole rows.
// Decoding is the same with a tile of one token: it streams the state, 16 bytes per lane. At the end the workgroup moves its
// channels' convolution windows on (the convolution, which reads the old ones, has finished by then). A sequence whose portion
// starts at position 0 starts from zero: slots need no clearing between owners.
#include "ds_hip.h"

#include <type_traits>

namespace {

constexpr int NT = 256;
constexpr float LOG2E = 1.4426950408889634f;

struct SelArgs {
  const void *x, *dt, *bc, *z, *cx;       // x, dt [T, C]; bc [T, B | C], z, cx [T, C]: columns, rows ld* apart
  int64_t ldbc, ldz, ldcx;
  const float *dt_bias, *a_log, *skip;    // [C], [C, N], [C]
  float* state;                           // [slots, C, NS]
  void* conv;                             // [slots, taps - 1, C]: last rows of cx, or null
  const int *cu, *start, *slots;
  void* out;                              // [T, C]
  int C, N, NS, taps, seqs;
};

// log(1 + e^v) to a few units in the last place: what adding 1 rounds off is put right by the last factor
__device__ __forceinline__ float softplus_f(float v) {
  const float u = __expf(-fabsf(v)), w = 1.f + u, d = w - 1.f;
  return fmaxf(v, 0.f) + (d == 0.f ? u : __logf(w) * (u * __builtin_amdgcn_rcpf(d)));
}
__device__ __forceinline__ float silu_f(float z) { return z * __builtin_amdgcn_rcpf(1.f + __expf(-z)); }

// Sum over groups of LP neighbouring lanes, in all of them
template <int LP>
__device__ __forceinline__ float group_sum(float v) {
  auto add = [&](auto sel) {
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), decltype(sel)::value, 0xf, 0xf, true));
  };
  add(std::integral_constant<int, 0xb1>{});                      // quad_perm: lane ^ 1
  add(std::integral_constant<int, 0x4e>{});                      // quad_perm: lane ^ 2
  if constexpr (LP >= 8) add(std::integral_constant<int, 0x141>{});   // row_half_mirror: the other quad of 8
  if constexpr (LP >= 16) add(std::integral_constant<int, 0x140>{});  // row_mirror: the other half of 16
  return v;
}

template <typename T, int LP, int NPL>
__global__ void __launch_bounds__(NT) selective_scan_kernel(SelArgs a) {
  constexpr int CH = NT / LP, NW = LP * NPL;               // channels; numbers per channel as they are laid out in LDS
  constexpr int TT = LP == 4 || NW > 128 ? 16 : 32;        // tokens of a tile
  constexpr int PER = TT * CH / NT;                        // (token, channel) pairs per thread
  __shared__ __attribute__((aligned(16))) f32x2 sx[TT][CH];  // step, step * x
  __shared__ __attribute__((aligned(16))) f32x2 sb[TT][NW];  // B, C
  __shared__ float sy[TT][CH];
  const int blocks = (a.C + CH - 1) / CH, id = xcd_remap(blockIdx.x, gridDim.x);
  const int seq = id / blocks, c0 = id % blocks * CH, tid = threadIdx.x;
  const int t0 = a.cu[seq], n = a.cu[seq + 1] - t0;
  if (n <= 0) return;
  const bool old = a.start[seq] > 0;
  // ---- this lane's numbers
  const int g = tid % LP, cl = tid / LP, c = min(c0 + cl, a.C - 1), n0 = g * NPL;
  const bool mine = c0 + cl < a.C;
  float* st = a.state + ((int64_t)a.slots[seq] * a.C + c) * a.NS + n0;
  float S[NPL], A[NPL];
#pragma unroll
  for (int i = 0; i < NPL; ++i) {
    const int k = min(n0 + i, a.N - 1);
    S[i] = 0.f;
    if (old) S[i] = st[k - n0];
    A[i] = n0 + i < a.N ? -expf(a.a_log[(int64_t)c * a.N + k]) * LOG2E : 0.f;
    if (n0 + i >= a.N) S[i] = 0.f;
  }
  // ---- what this thread stages and writes: tokens (tid / CH) + PR j, channel tid % CH
  constexpr int PR = NT / CH;
  const int wc = c0 + tid % CH, wcc = min(wc, a.C - 1), wt = tid / CH;
  const float bias = a.dt_bias[wcc], skip = a.skip[wcc];
  T xr[PER], dr[PER], zr[PER];
  constexpr int BPER = (TT * NW + NT - 1) / NT;
  T br[BPER], cr[BPER];
  auto fetch = [&](int k0) {
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int64_t t = t0 + min(k0 + wt + PR * j, n - 1);
      xr[j] = ((const T*)a.x)[t * a.C + wcc];
      dr[j] = ((const T*)a.dt)[t * a.C + wcc];
      zr[j] = ((const T*)a.z)[t * a.ldz + wcc];
    }
#pragma unroll
    for (int j = 0; j < BPER; ++j) {
      const int e = tid + NT * j;
      const T* p = (const T*)a.bc + (int64_t)(t0 + min(k0 + min(e / NW, TT - 1), n - 1)) * a.ldbc + min(e % NW, a.N - 1);
      br[j] = p[0];
      cr[j] = p[a.N];
    }
  };
  fetch(0);
  for (int k0 = 0; k0 < n; k0 += TT) {
    float xs[PER], zs[PER];
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      xs[j] = (float)xr[j];
      zs[j] = (float)zr[j];
      const float step = softplus_f((float)dr[j] + bias);
      sx[wt + PR * j][tid % CH] = f32x2{step, step * xs[j]};
    }
#pragma unroll
    for (int j = 0; j < BPER; ++j) {
      const int e = tid + NT * j;
      if (e < TT * NW) sb[e / NW][e % NW] = e % NW < a.N ? f32x2{(float)br[j], (float)cr[j]} : f32x2{0.f, 0.f};
    }
    __syncthreads();
    if (k0 + TT < n) fetch(k0 + TT);
    const int m = min(TT, n - k0);
    auto token = [&](int t) {
      const f32x2 sd = sx[t][cl];
      float y = 0.f;
#pragma unroll
      for (int i = 0; i < NPL; ++i) {
        const f32x2 b = sb[t][n0 + i];
        S[i] = fmaf(__builtin_amdgcn_exp2f(sd[0] * A[i]), S[i], sd[1] * b[0]);
        y = fmaf(S[i], b[1], y);
      }
      return group_sum<LP>(y);
    };
    int t = 0;
    for (; t + LP <= m; t += LP) {
      float keep = 0.f;
#pragma unroll
      for (int i = 0; i < LP; ++i) {
        const float y = token(t + i);
        keep = g == i ? y : keep;
      }
      sy[t + g][cl] = keep;
    }
    for (; t < m; ++t) {
      const float y = token(t);
      if (g == 0) sy[t][cl] = y;
    }
    __syncthreads();
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int r = wt + PR * j;
      const float y = fmaf(skip, xs[j], sy[r][tid % CH]);
      if (r < m && wc < a.C) ((T*)a.out)[(int64_t)(t0 + k0 + r) * a.C + wc] = (T)(y * silu_f(zs[j]));
    }
  }
  if (mine) {
#pragma unroll
    for (int i = 0; i < NPL; ++i)
      if (n0 + i < a.N) st[i] = S[i];
  }
  // ---- convolution windows: the last taps - 1 of [old window | the portion's inputs]
  if (a.conv && tid < CH && c0 + tid < a.C) {
    const int ch = c0 + tid, w = a.taps - 1;
    T* cs = (T*)a.conv + (int64_t)a.slots[seq] * w * a.C + ch;
    for (int j = 0; j < w; ++j) {
      const int src = n + j;
      T v = (T)0.f;
      if (src >= w) v = ((const T*)a.cx)[(int64_t)(t0 + src - w) * a.ldcx + ch];
      else if (old) v = cs[(int64_t)src * a.C];
      cs[(int64_t)j * a.C] = v;  // ascending: src > j, so nothing is overwritten before it is read
    }
  }
}

template <typename T, int LP>
int launch(const SelArgs& a, hipStream_t st) {
  constexpr int CH = NT / LP;
  const int64_t grid = (int64_t)((a.C + CH - 1) / CH) * a.seqs;
  if (grid > INT32_MAX) return (int)hipErrorInvalidValue;
  const int need = (a.N + LP - 1) / LP;
#define GO(NPL)                                                                                                    \
  {                                                                                                                \
    hipLaunchKernelGGL((selective_scan_kernel<T, LP, NPL>), dim3((unsigned)grid), dim3(NT), 0, st, a);             \
    DS_CHECK_LAUNCH();                                                                                             \
    return 0;                                                                                                      \
  }
  if (need <= 1) GO(1)
  if (need <= 2) GO(2)
  if (need <= 3) GO(3)
  if (need <= 4) GO(4)
  if (need <= 6) GO(6)
  if (need <= 8) GO(8)
  if constexpr (LP == 16) {
    if (need <= 16) GO(16)
  }
#undef GO
  return (int)hipErrorInvalidValue;
}

template <typename T>
int choose(const SelArgs& a, bool decode, hipStream_t st) {
  // waves with 4 lanes per channel; as few lanes as cover the chip's 1024 SIMDs
  const int64_t waves = (int64_t)a.C * a.seqs / 16;
  if (a.N <= 32 && (decode || waves >= 1024)) return launch<T, 4>(a, st);
  if (a.N <= 64 && (decode || waves >= 512)) return launch<T, 8>(a, st);
  return launch<T, 16>(a, st);
}

}  // namespace

// Numbers per channel a kernel instance holds
extern "C" int ds_selective_scan_max() { return 256; }

// x, dt [T, C] and, ldbc / ldz / ldcx elements from row to row, bc [T, B | C (N each)], z [T, C], cx [T, C]; state
// [slots, C, NS]; conv [slots, taps - 1, C] or null. `longest`: most new tokens of a sequence
extern "C" int ds_selective_scan(const void* x, const void* dt, const void* bc, int64_t ldbc, const void* z, int64_t ldz,
                                 const float* dt_bias, const float* a_log, const float* skip, float* state, const void* cx,
                                 int64_t ldcx, void* conv, const int* cu, const int* start, const int* slots, void* out, int seqs,
                                 int longest, int C, int N, int NS, int taps, int dtype, hipStream_t st) {
  if (seqs <= 0) return 0;
  if (C <= 0 || N <= 0 || N > ds_selective_scan_max() || NS < N || taps < 1 || (conv && (taps < 2 || !cx)))
    return (int)hipErrorInvalidValue;
  const SelArgs a{x, dt, bc, z, cx, ldbc, ldz, ldcx, dt_bias, a_log, skip, state, conv, cu, start, slots, out, C, N, NS, taps, seqs};
  if (dtype == DS_F32) return choose<float>(a, longest <= 4, st);
  if (dtype == DS_BF16) return choose<bf16>(a, longest <= 4, st);
  return (int)hipErrorInvalidValue;
}
