// Shared by the kernels of recurrences with a scalar decay per head (decayed_scan.hip: token by token, decayed_chunk.hip:
// by chunks).
#pragma once
#include "ds_hip.h"

namespace {

constexpr int Z_COLS = 32;

// Fused projection row of `rows` columns: q, k [Hk heads of dk], v [H heads of dv] start at columns q, k, v; `channels`
// columns from `conv` on pass a convolution of `taps`; dt: first of H step-size columns, or -1.
struct ScanDims {
  int rows, q, k, v, Hk, H, dk, dv, taps, conv, channels, dt;
  int64_t T;  // tokens of the batch
  __host__ __device__ int dks() const { return (dk + 7) & ~7; }  // widths as q, k, the state (dks) and v (dvs) are stored
  __host__ __device__ int dvs() const { return (dv + 7) & ~7; }
  // head by head, [heads, T, width]: tiles of a head's rows spread over the memory channels whatever the head count
  __host__ __device__ int64_t q_at(int g, int64_t t) const { return ((int64_t)g * T + t) * dks(); }
  __host__ __device__ int64_t k_at(int g, int64_t t) const { return ((int64_t)(Hk + g) * T + t) * dks(); }
  // normaliser of the columns around `col`: a slot holds a copy for every Z_COLS value columns, [H, copies, dks]
  __host__ __device__ int zc() const { return (dv + Z_COLS - 1) / Z_COLS; }
  __host__ __device__ int64_t z_at(int64_t slot, int h, int col) const { return ((slot * H + h) * zc() + col / Z_COLS) * dks(); }
  __host__ __device__ int64_t v_at(int h, int64_t t) const { return ((int64_t)h * T + t) * dvs(); }
};

// A channel's convolution window: the last taps - 1 inputs of [old window | the portion's inputs].
template <typename T>
__device__ __forceinline__ void advance_channel(T* cs, const T* proj, int64_t t0, int n, const ScanDims& D, bool fresh, int c) {
  for (int j = 0; j < D.taps - 1; ++j) {
    const int src = n + j;  // index in [old (taps-1) | new (n)]
    T x = (T)0.f;
    if (src >= D.taps - 1) x = proj[(t0 + src - (D.taps - 1)) * D.rows + D.conv + c];
    else if (!fresh) x = cs[(int64_t)src * D.channels + c];
    cs[(int64_t)j * D.channels + c] = x;  // ascending: src > j, so nothing is overwritten before it is read
  }
}

// Windows of head h's value channels, and of its group's q / k channels if it is the group's first head
template <typename T>
__device__ __forceinline__ void advance_windows(T* cs, const T* proj, int64_t t0, int n, const ScanDims& D, bool fresh, int h) {
  const int rep = D.H / D.Hk, g = h / rep;
  for (int c = threadIdx.x; c < D.dv; c += blockDim.x)
    advance_channel(cs, proj, t0, n, D, fresh, D.v - D.conv + h * D.dv + c);
  if (h % rep == 0)
    for (int c = threadIdx.x; c < 2 * D.dk; c += blockDim.x)
      advance_channel(cs, proj, t0, n, D, fresh, (c < D.dk ? D.q : D.k - D.dk) - D.conv + g * D.dk + c);
}

static inline bool scan_dims_ok(const ScanDims& D) {
  return D.Hk > 0 && D.H > 0 && D.H % D.Hk == 0 && D.dk > 0 && D.dv > 0 && D.dk <= 512 && D.taps >= 1 && D.H <= 65535;
}

}  // namespace
