// Shared by the gated-delta-rule kernels (delta_rule.hip: token by token, delta_chunk.hip: by chunks).
#pragma once
#include "ds_hip.h"

namespace {

__device__ __forceinline__ float silu(float x) { return x / (1.f + expf(-x)); }

// Elements c, c + 1 of a row of `width` (c even); where c lies beyond the row, some element of it (the caller drops it).
// PAIR: rows are even and pair-aligned, so this is one unconditional access.
template <bool PAIR, typename T>
__device__ __forceinline__ void load2(const T* row, int c, int width, float (&v)[2]) {
  typedef T T2 __attribute__((ext_vector_type(2)));
  if constexpr (PAIR) {
    const T2 a = *reinterpret_cast<const T2*>(row + min(c, width - 2));
    v[0] = (float)a[0];
    v[1] = (float)a[1];
  } else {
    v[0] = (float)row[min(c, width - 1)];
    v[1] = (float)row[min(c + 1, width - 1)];
  }
}
template <bool PAIR, typename T>
__device__ __forceinline__ void store2(T* row, int c, int width, const float (&v)[2]) {
  typedef T T2 __attribute__((ext_vector_type(2)));
  if constexpr (PAIR) {
    T2 a;
    a[0] = (T)v[0];
    a[1] = (T)v[1];
    if (c < width) *reinterpret_cast<T2*>(row + c) = a;
  } else {
    if (c < width) row[c] = (T)v[0];
    if (c + 1 < width) row[c + 1] = (T)v[1];
  }
}

struct DeltaDims {
  int Hk, H, dk, dv, taps;
  int64_t T;  // tokens of the batch
  __host__ __device__ int channels() const { return 2 * Hk * dk + H * dv; }
  __host__ __device__ int dks() const { return (dk + 3) & ~3; }  // key width as q, k and the state are stored (zero padded)
  // q, k (and v, the read-out) are kept head by head, [heads, T, width]: a head's rows are contiguous, and tiles of them
  // spread over the memory channels whatever the head count
  __host__ __device__ int64_t q_at(int hk, int64_t t) const { return ((int64_t)hk * T + t) * dks(); }
  __host__ __device__ int64_t k_at(int hk, int64_t t) const { return ((int64_t)(Hk + hk) * T + t) * dks(); }
  __host__ __device__ int64_t v_at(int h, int64_t t) const { return ((int64_t)h * T + t) * dv; }
  __host__ __device__ int row() const { return channels() + H * dv + 2 * H; }
};

// Window of one channel: the last taps-1 inputs of [old window | the portion's inputs].
template <typename T>
__device__ __forceinline__ void advance_window(T* cs, const T* proj, int64_t t0, int n, int NP, int C, int taps, bool fresh,
                                               int c) {
  for (int j = 0; j < taps - 1; ++j) {
    const int src = n + j;  // index in [old (taps-1) | new (n)]
    T x = (T)0.f;
    if (src >= taps - 1) x = proj[(t0 + src - (taps - 1)) * NP + c];
    else if (!fresh) x = cs[(int64_t)src * C + c];
    cs[(int64_t)j * C + c] = x;  // ascending: src > j, so nothing is overwritten before it is read
  }
}

// Convolution windows of head h's own channels (its values, and the group's q / k if it is the group's first head).
template <typename T>
__device__ __forceinline__ void advance_head(T* cs, const T* proj, int64_t t0, int n, const DeltaDims& D, bool fresh, int h) {
  const int NP = D.row(), C = D.channels(), rep = D.H / D.Hk;
  for (int c = threadIdx.x; c < D.dv; c += blockDim.x)
    advance_window(cs, proj, t0, n, NP, C, D.taps, fresh, 2 * D.Hk * D.dk + h * D.dv + c);
  if (h % rep == 0)
    for (int c = threadIdx.x; c < 2 * D.dk; c += blockDim.x)
      advance_window(cs, proj, t0, n, NP, C, D.taps, fresh,
                     (c < D.dk ? 0 : (D.Hk - 1) * D.dk) + (h / rep) * D.dk + c);
}

static inline bool dims_ok(const DeltaDims& D) {
  return D.Hk > 0 && D.H > 0 && D.H % D.Hk == 0 && D.dk > 0 && D.dv > 0 && D.dk <= 256 && D.dv <= 256 && D.taps >= 1;
}

}  // namespace
