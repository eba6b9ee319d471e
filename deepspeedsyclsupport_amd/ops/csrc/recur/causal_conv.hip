// Short causal convolution per channel with bias and silu, over a ragged batch, CDNA4 (gfx950). Inputs may be columns of a wider
// matrix; those before a portion come from the sequence's slot of convolution windows. A sequence whose portion starts at position
// 0 has zeros before it. The window of a portion of one token moves on here, where it is in registers; other portions are shared
// by several waves, and the recurrence behind the convolution moves theirs on.
//
// HBM-bound: a lane has up to 8 channels of a tile of consecutive tokens, all its inputs in flight at once.
#include "ds_hip.h"

namespace {

template <typename T, int V>
__device__ __forceinline__ void ldv(const T* p, float (&v)[V]) {
  if constexpr (V == 8) Vec8<T>::load(p, v);
  else v[0] = (float)p[0];
}
template <typename T, int V>
__device__ __forceinline__ void stv(T* p, const float (&v)[V]) {
  if constexpr (V == 8) Vec8<T>::store(p, v);
  else p[0] = (T)v[0];
}

struct ConvArgs {
  const void* x;       // [T, C], rows ld apart
  int64_t ld;
  const float* w;      // [C, taps], last column: the current token
  const float* b;      // [C]
  void* state;         // [slots, taps - 1, C]
  const int *seq_ids, *cu, *start, *slots;
  void* out;           // [T, C]
  int tokens, C, taps;
};

// TAPS: filter length, the tile's inputs in registers; 0: any length, inputs read per tap. V channels per lane; TILE: consecutive
// tokens of a wave (a few decodes spread over the chip one by one).
template <typename T, int TAPS, int V, int TILE>
__global__ void __launch_bounds__(256) causal_conv_kernel(ConvArgs a) {
  const int lane = threadIdx.x & 63, parts = (a.C + 64 * V - 1) / (64 * V), taps = TAPS ? TAPS : a.taps;
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6), tl = item / parts * TILE;
  const int c = (int)(item % parts) * 64 * V + lane * V;
  if (tl >= a.tokens || c >= a.C) return;
  const T* x = (const T*)a.x + c;
  const float* w = a.w + (int64_t)c * taps;
  float bias[V];
#pragma unroll
  for (int e = 0; e < V; ++e) bias[e] = a.b[c + e];
  const int t_hi = min((int)tl + TILE, a.tokens);
  for (int ta = (int)tl; ta < t_hi;) {  // runs of tokens of one sequence
    const int seq = a.seq_ids[ta], first = a.cu[seq], tb = min(t_hi, a.cu[seq + 1]), n = tb - ta, j0 = ta - first;
    T* const window = taps == 1 ? nullptr : (T*)a.state + (int64_t)a.slots[seq] * (taps - 1) * a.C + c;
    const T* old = a.start[seq] == 0 ? nullptr : window;
    const bool lone = window && a.cu[seq + 1] - first == 1;
    // the input at place j of the portion (negative: before it); zero tells that there is none
    auto input = [&](int j, float (&v)[V]) {
      const bool none = j < 0 && !old;
      ldv<T, V>(j >= 0 || none ? x + (int64_t)(first + max(j, 0)) * a.ld : old + (int64_t)(j + taps - 1) * a.C, v);
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] = none ? 0.f : v[e];
    };
    float y[TILE][V];
    if constexpr (TAPS != 0) {
      float in[TILE + TAPS - 1][V], cw[V][TAPS];
#pragma unroll
      for (int i = 0; i < TILE + TAPS - 1; ++i) input(j0 + min(i, n + TAPS - 2) - (TAPS - 1), in[i]);
#pragma unroll
      for (int e = 0; e < V; ++e)
#pragma unroll
        for (int i = 0; i < TAPS; ++i) cw[e][i] = w[e * TAPS + i];
#pragma unroll
      for (int t = 0; t < TILE; ++t)
#pragma unroll
        for (int e = 0; e < V; ++e) {
          float acc = bias[e];
#pragma unroll
          for (int i = 0; i < TAPS; ++i) acc = fmaf(cw[e][i], in[t + i][e], acc);
          y[t][e] = acc;
        }
      if (lone) {
#pragma unroll
        for (int i = 1; i < TAPS; ++i) stv<T, V>(window + (int64_t)(i - 1) * a.C, in[i]);
      }
    } else {
#pragma unroll
      for (int t = 0; t < TILE; ++t)
#pragma unroll
        for (int e = 0; e < V; ++e) y[t][e] = bias[e];
      for (int i = 0; i < taps; ++i) {
#pragma unroll
        for (int t = 0; t < TILE; ++t) {
          float v[V];
          input(j0 + min(t, n - 1) - (taps - 1) + i, v);
#pragma unroll
          for (int e = 0; e < V; ++e) y[t][e] = fmaf(w[e * taps + i], v[e], y[t][e]);
        }
      }
      if (lone) {  // (ascending: a row is read before it is written)
        for (int i = 1; i < taps; ++i) {
          float v[V];
          input(i - (taps - 1), v);
          stv<T, V>(window + (int64_t)(i - 1) * a.C, v);
        }
      }
    }
#pragma unroll
    for (int t = 0; t < TILE; ++t) {
      if (t >= n) break;
#pragma unroll
      for (int e = 0; e < V; ++e) y[t][e] = y[t][e] / (1.f + expf(-y[t][e]));
      stv<T, V>((T*)a.out + (int64_t)(ta + t) * a.C + c, y[t]);
    }
    ta = tb;
  }
}

template <typename T, int V, int TILE>
int launch(const ConvArgs& a, hipStream_t st) {
  const int64_t items = (int64_t)((a.tokens + TILE - 1) / TILE) * ((a.C + 64 * V - 1) / (64 * V));
  const dim3 grid((unsigned)((items + 3) / 4));
  switch (a.taps) {
    case 2: hipLaunchKernelGGL((causal_conv_kernel<T, 2, V, TILE>), grid, dim3(256), 0, st, a); break;
    case 3: hipLaunchKernelGGL((causal_conv_kernel<T, 3, V, TILE>), grid, dim3(256), 0, st, a); break;
    case 4: hipLaunchKernelGGL((causal_conv_kernel<T, 4, V, TILE>), grid, dim3(256), 0, st, a); break;
    default: hipLaunchKernelGGL((causal_conv_kernel<T, 0, V, TILE>), grid, dim3(256), 0, st, a);
  }
  DS_CHECK_LAUNCH();
  return 0;
}

template <typename T>
int conv(const ConvArgs& a, bool vec, hipStream_t st) {
  if (!vec) return launch<T, 1, 8>(a, st);
  return a.tokens <= 512 ? launch<T, 8, 1>(a, st) : launch<T, 8, 8>(a, st);
}

}  // namespace

// x [tokens, C], rows ld elements apart -> out [tokens, C] = silu(conv(x) + b); state [slots, taps - 1, C] (unused with one tap)
extern "C" int ds_causal_conv(const void* x, int64_t ld, const float* w, const float* b, void* state, const int* seq_ids,
                              const int* cu, const int* start, const int* slots, void* out, int tokens, int C, int taps,
                              int dtype, hipStream_t st) {
  if (tokens <= 0) return 0;
  if (C <= 0 || taps < 1 || ld < C || (taps > 1 && !state)) return (int)hipErrorInvalidValue;
  const ConvArgs a{x, ld, w, b, state, seq_ids, cu, start, slots, out, tokens, C, taps};
  const bool vec = C % 8 == 0 && ld % 8 == 0 && (((uintptr_t)x | (uintptr_t)state) & 15) == 0;
  if (dtype == DS_F32) return conv<float>(a, vec, st);
  if (dtype == DS_BF16) return conv<bf16>(a, vec, st);
  return (int)hipErrorInvalidValue;
}
