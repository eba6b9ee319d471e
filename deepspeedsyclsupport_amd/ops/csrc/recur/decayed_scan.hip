// Recurrences with a scalar decay per head (state-space duality, linear attention with constant decays), CDNA4 (gfx950).
//
// Per head, with a state S [dk, dv] in fp32 that starts at zero:
//     S <- a S + b k v^T;   o = c S^T q + D v
// with b = softplus(dt + dt_bias), a = exp(-exp(A_log) b) per token, or any a and b per token (exp_gates.hip), or b = 1 and a
// constant a; c is a constant. q, k and v are columns of a fused projection row. Several heads may share q and k. With a
// normaliser, z <- a z + b k runs beside the state and o becomes c S^T q / (max(|c z . q|, floor) + 1e-6), floor per token.
//
//  * prepare: q, k and v after (optionally) a causal convolution with bias and silu. A lane per few channels of a tile of
//    consecutive tokens; inputs before the portion come from the sequence's state slot. Step sizes and log decays leave it in
//    fp32, q / k / v in the storage type (they are activations).
//  * split: q, k and v as they are, with (optionally) pairs of columns of q and k turned to their positions. In 16-bit storage
//    the turned ones leave as the sum of two terms: what enters a recurrence is not rounded to 16 bits again.
//  * recur: one workgroup per (sequence, head, 64 value columns), the state in registers while the portion's tokens pass
//    one by one: decoding, short portions, and everything in fp32 models. It also moves the convolution's windows on
//    (prepare, which reads the old ones, has finished by then).
// A sequence whose portion starts at position 0 starts from zero: slots need no clearing between owners.
#include "decayed_scan.h"

namespace {

constexpr int TILE = 8;  // consecutive tokens a prepare wave walks

template <typename T, int V>
__device__ __forceinline__ void ldv(const T* p, float (&v)[V]) {
  typedef T TV __attribute__((ext_vector_type(V == 1 ? 2 : V)));
  if constexpr (V == 1) {
    v[0] = (float)p[0];
  } else {
    const TV a = *reinterpret_cast<const TV*>(p);
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] = (float)a[i];
  }
}
template <typename T, int V>
__device__ __forceinline__ void stv(T* p, const float (&v)[V]) {
  typedef T TV __attribute__((ext_vector_type(V == 1 ? 2 : V)));
  if constexpr (V == 1) {
    p[0] = (T)v[0];
  } else {
    TV a;
#pragma unroll
    for (int i = 0; i < V; ++i) a[i] = (T)v[i];
    *reinterpret_cast<TV*>(p) = a;
  }
}

// TAPS: filter length (1: no convolution), the tile's inputs in registers; 0: any length, inputs read per tap.
template <typename T, int TAPS, int V>
__global__ void __launch_bounds__(256) scan_prepare_kernel(
    const T* __restrict__ proj, const float* __restrict__ conv_w, const float* __restrict__ conv_b,
    const T* __restrict__ conv_state, const float* __restrict__ a_log, const float* __restrict__ dt_bias,
    const int* __restrict__ seq_ids, const int* __restrict__ cu, const int* __restrict__ start,
    const int* __restrict__ slots, T* __restrict__ qk, T* __restrict__ v_out, float* __restrict__ gb, int tile, ScanDims D) {
  constexpr int CW = 64 * V;  // channels of a wave
  const int nq = (D.Hk * D.dk + CW - 1) / CW, nv = (D.H * D.dv + CW - 1) / CW, parts = 2 * nq + nv + (gb ? 1 : 0);
  const int lane = threadIdx.x & 63;
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  const int tokens = (int)D.T, part = (int)(item % parts);
  const int64_t tl = item / parts * tile;
  if (tl >= tokens) return;
  const int t_lo = (int)tl, t_hi = min(t_lo + tile, tokens);
  if (part == 2 * nq + nv) {  // step sizes and log decays
    for (int t = t_lo; t < t_hi; ++t)
      for (int h = lane; h < D.H; h += 64) {
        const float z = (float)proj[(int64_t)t * D.rows + D.dt + h] + dt_bias[h];
        const float b = z > 20.f ? z : log1pf(expf(z));
        gb[((int64_t)t * 2) * D.H + h] = -expf(a_log[h]) * b;
        gb[((int64_t)t * 2 + 1) * D.H + h] = b;
      }
    return;
  }
  const int kind = part < nq ? 0 : part < 2 * nq ? 1 : 2;  // q, k, v
  const int width = kind == 2 ? D.dv : D.dk, total = width * (kind == 2 ? D.H : D.Hk);
  const int c = (part - (kind == 2 ? 2 * nq : kind * nq)) * CW + lane * V;
  if (c >= total) return;
  const int col = (kind == 0 ? D.q : kind == 1 ? D.k : D.v) + c, ch = col - D.conv, taps = TAPS ? TAPS : D.taps;
  const int head = c / width, in = c % width;  // (V divides the width)
  float bias[V];
#pragma unroll
  for (int e = 0; e < V; ++e) bias[e] = conv_b ? conv_b[ch + e] : 0.f;
  for (int ta = t_lo; ta < t_hi;) {  // runs of tokens of one sequence
    const int seq = seq_ids[ta], first = cu[seq], tb = min(t_hi, cu[seq + 1]), n = tb - ta, j0 = ta - first;
    const T* cs = start[seq] == 0 || taps == 1 ? nullptr : conv_state + (int64_t)slots[seq] * (taps - 1) * D.channels + ch;
    // the convolution's input at place j of the portion (negative: before it); zero tells that there is none
    auto row = [&](int j, float& zero) {
      zero = j >= 0 || cs ? 1.f : 0.f;
      return j >= 0 || !cs ? proj + (int64_t)(first + max(j, 0)) * D.rows + col : cs + (int64_t)(j + taps - 1) * D.channels;
    };
    float y[TILE][V];
    if constexpr (TAPS == 1) {
#pragma unroll
      for (int t = 0; t < TILE; ++t) ldv<T, V>(proj + (int64_t)(ta + min(t, n - 1)) * D.rows + col, y[t]);
      if (conv_w) {
#pragma unroll
        for (int t = 0; t < TILE; ++t)
#pragma unroll
          for (int e = 0; e < V; ++e) y[t][e] = fmaf(conv_w[ch + e], y[t][e], bias[e]);
      }
    } else if constexpr (TAPS != 0) {
      float x[TILE + TAPS - 1][V], cw[V][TAPS];
#pragma unroll
      for (int i = 0; i < TILE + TAPS - 1; ++i) {
        float zero;
        const T* r = row(j0 + min(i, n + TAPS - 2) - (TAPS - 1), zero);
        ldv<T, V>(r, x[i]);
#pragma unroll
        for (int e = 0; e < V; ++e) x[i][e] *= zero;
      }
#pragma unroll
      for (int e = 0; e < V; ++e)
#pragma unroll
        for (int i = 0; i < TAPS; ++i) cw[e][i] = conv_w[(int64_t)(ch + e) * TAPS + i];
#pragma unroll
      for (int t = 0; t < TILE; ++t)
#pragma unroll
        for (int e = 0; e < V; ++e) {
          float acc = bias[e];
#pragma unroll
          for (int i = 0; i < TAPS; ++i) acc = fmaf(cw[e][i], x[t + i][e], acc);
          y[t][e] = acc;
        }
    } else {
#pragma unroll
      for (int t = 0; t < TILE; ++t)
#pragma unroll
        for (int e = 0; e < V; ++e) y[t][e] = bias[e];
      for (int i = 0; i < taps; ++i) {
#pragma unroll
        for (int t = 0; t < TILE; ++t) {
          float zero, x[V];
          const T* r = row(j0 + min(t, n - 1) - (taps - 1) + i, zero);
          ldv<T, V>(r, x);
#pragma unroll
          for (int e = 0; e < V; ++e) y[t][e] = fmaf(conv_w[(int64_t)(ch + e) * taps + i], x[e] * zero, y[t][e]);
        }
      }
    }
#pragma unroll
    for (int t = 0; t < TILE; ++t) {
      if (t >= n) break;
#pragma unroll
      for (int e = 0; e < V; ++e) y[t][e] = y[t][e] / (1.f + expf(-y[t][e]));
      T* dst = kind == 2 ? v_out + D.v_at(head, ta + t) : qk + (kind ? D.k_at(head, ta + t) : D.q_at(head, ta + t));
      stv<T, V>(dst + in, y[t]);
    }
    ta = tb;
  }
}

// One workgroup per token: the row's q, k and v head by head, pairs (i, i + half) of the first 2 half columns of q and k turned
// by the token's angles cs [half, 2]; `term` (0: none): from the first terms of q and k to what rounding them left out
template <typename T, int V>
__global__ void __launch_bounds__(256) scan_split_kernel(const T* __restrict__ proj, const float* __restrict__ cs, int half,
                                                         T* __restrict__ qk, T* __restrict__ v_out, int64_t term, ScanDims D) {
  const int t = blockIdx.x, tid = threadIdx.x;
  const T* row = proj + (int64_t)t * D.rows;
  const float* a = cs + (int64_t)t * half * 2;
  const int per = (D.dk - half) / V, hv = half / V;  // a head's pairs, then its columns without one
  for (int i = tid; i < 2 * D.Hk * per; i += 256) {
    const int g = i / per, j = i % per;
    const T* src = row + (g < D.Hk ? D.q + g * D.dk : D.k + (g - D.Hk) * D.dk);
    T* dst = qk + D.q_at(g, t);  // (k's heads lie behind q's)
    if (j < hv) {
      const int c = j * V;
      float u[V], w[V], x[V], y[V];
      ldv<T, V>(src + c, u);
      ldv<T, V>(src + half + c, w);
#pragma unroll
      for (int e = 0; e < V; ++e) {
        const float co = a[2 * (c + e)], si = a[2 * (c + e) + 1];
        x[e] = u[e] * co - w[e] * si;
        y[e] = w[e] * co + u[e] * si;
      }
      stv<T, V>(dst + c, x);
      stv<T, V>(dst + half + c, y);
      if (term) {
#pragma unroll
        for (int e = 0; e < V; ++e) {
          x[e] -= (float)(T)x[e];
          y[e] -= (float)(T)y[e];
        }
        stv<T, V>(dst + term + c, x);
        stv<T, V>(dst + term + half + c, y);
      }
    } else {
      const int c = half + j * V;
      float u[V];
      ldv<T, V>(src + c, u);
      stv<T, V>(dst + c, u);
      if (term) {
#pragma unroll
        for (int e = 0; e < V; ++e) u[e] = 0.f;
        stv<T, V>(dst + term + c, u);
      }
    }
  }
  const int pv = D.dv / V;
  for (int i = tid; i < D.H * pv; i += 256) {
    const int h = i / pv, c = i % pv * V;
    float u[V];
    ldv<T, V>(row + D.v + h * D.dv + c, u);
    stv<T, V>(v_out + D.v_at(h, t) + c, u);
  }
}

constexpr int LPC = 8;     // lanes per value column: lane p holds key rows 4 (p + LPC i) + 0..3
constexpr int COLS = 64;   // value columns per workgroup

// NORM: with a normaliser; TWO: q and k of two terms
template <typename T, int NV, bool NORM, bool TWO>
__global__ void __launch_bounds__(LPC * COLS) scan_recur_kernel(
    const T* __restrict__ qk, const T* __restrict__ v, const float* __restrict__ gb, const float* __restrict__ log_decay,
    const float* __restrict__ skip, float scale, const T* __restrict__ proj, float* __restrict__ state,
    float* __restrict__ zstate, const float* __restrict__ floors, T* __restrict__ conv_state, const int* __restrict__ list,
    int lstride, const int* __restrict__ cu, const int* __restrict__ start, const int* __restrict__ slots, T* __restrict__ out,
    ScanDims D) {
  const int seq = list[blockIdx.x * lstride], h = blockIdx.y, g = h / (D.H / D.Hk), tid = threadIdx.x;
  const int64_t t0 = cu[seq];
  const int n = cu[seq + 1] - (int)t0, col = blockIdx.z * COLS + tid / LPC, p = tid % LPC, dks = D.dks();
  const bool fresh = start[seq] == 0, on = col < D.dv;
  float* st = state + (((int64_t)slots[seq] * D.H + h) * D.dv + min(col, D.dv - 1)) * dks;
  // every Z_COLS columns have a copy of the normaliser, so that no workgroup reads what another one writes
  float* zt = NORM ? zstate + D.z_at(slots[seq], h, min(col, D.dv - 1)) : nullptr;
  f32x4 S[NV], Z[NORM ? NV : 1];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int k = 4 * (p + LPC * i);
    S[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (!fresh && k < dks) S[i] = *reinterpret_cast<const f32x4*>(st + k);
    if constexpr (NORM) {
      Z[i] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (!fresh && k < dks) Z[i] = *reinterpret_cast<const f32x4*>(zt + k);
    }
  }
  // (every column of a copy has read it before its first one writes it: they are of one workgroup)
  if constexpr (NORM) __syncthreads();
  const float sk = skip ? skip[h] : 0.f, ld = log_decay ? log_decay[h] : 0.f;
  const int64_t term = 2 * D.Hk * D.T * dks;
  for (int t = 0; t < n; ++t) {
    const int64_t tok = t0 + t;
    const float a = expf(gb ? gb[tok * 2 * D.H + h] : ld), b = gb ? gb[(tok * 2 + 1) * D.H + h] : 1.f;
    const float vv = (float)v[D.v_at(h, tok) + min(col, D.dv - 1)], u = b * vv;
    float o = 0.f, zq = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int k = 4 * (p + LPC * i), kc = min(k, dks - 4);
      float kf[4], qf[4];
      ldv<T, 4>(qk + D.k_at(g, tok) + kc, kf);
      ldv<T, 4>(qk + D.q_at(g, tok) + kc, qf);
      if constexpr (TWO) {
        float kl[4], ql[4];
        ldv<T, 4>(qk + term + D.k_at(g, tok) + kc, kl);
        ldv<T, 4>(qk + term + D.q_at(g, tok) + kc, ql);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          kf[e] += kl[e];
          qf[e] += ql[e];
        }
      }
      const float z = k < dks ? 1.f : 0.f;  // rows past the width stay zero
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[i][e] = fmaf(kf[e] * z, u, a * S[i][e]);
        o = fmaf(S[i][e], qf[e], o);
        if constexpr (NORM) {
          Z[i][e] = fmaf(kf[e] * z, b, a * Z[i][e]);
          zq = fmaf(Z[i][e], qf[e], zq);
        }
      }
    }
#pragma unroll
    for (int d = 1; d < LPC; d <<= 1) {
      o += __shfl_xor(o, d, 64);
      if constexpr (NORM) zq += __shfl_xor(zq, d, 64);
    }
    o *= scale;
    if constexpr (NORM) o /= fmaxf(fabsf(zq * scale), floors[tok * D.H + h]) + 1e-6f;
    if (on && p == 0) out[(tok * D.H + h) * D.dv + col] = (T)fmaf(sk, vv, o);
  }
  if (on) {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int k = 4 * (p + LPC * i);
      if (k < dks) *reinterpret_cast<f32x4*>(st + k) = S[i];
      if constexpr (NORM) {
        if (k < dks && col % Z_COLS == 0) *reinterpret_cast<f32x4*>(zt + k) = Z[i];
      }
    }
  }
  if (blockIdx.z == 0 && D.taps > 1)
    advance_windows(conv_state + (int64_t)slots[seq] * (D.taps - 1) * D.channels, proj, t0, n, D, fresh, h);
}

template <typename T>
int recur(const void* qk, const void* v, const float* gb, const float* log_decay, const float* skip, float scale,
          const void* proj, float* state, float* zstate, const float* floors, void* conv_state, int terms, const int* list, int nlist, int lstride, const int* cu, const int* start,
          const int* slots, void* out, const ScanDims& D, hipStream_t st) {
  const dim3 grid(nlist, D.H, (D.dv + COLS - 1) / COLS);
  const int nt = D.dv >= COLS ? LPC * COLS : (LPC * D.dv + 63) / 64 * 64, nv = (D.dks() / 4 + LPC - 1) / LPC;
#define RUN(NV, NORM, TWO)                                                                                                \
  hipLaunchKernelGGL((scan_recur_kernel<T, NV, NORM, TWO>), grid, dim3(nt), 0, st, (const T*)qk, (const T*)v, gb, log_decay,   \
                     skip, scale, (const T*)proj, state, zstate, floors, (T*)conv_state, list, lstride, cu, start, slots, \
                     (T*)out, D)
#define GO(NV)                                 \
  {                                            \
    if (zstate) RUN(NV, true, false);          \
    else if (terms == 2) RUN(NV, false, true); \
    else RUN(NV, false, false);                \
  }
  if (nv <= 1) GO(1)
  else if (nv <= 2) GO(2)
  else if (nv <= 4) GO(4)
  else if (nv <= 8) GO(8)
  else GO(16)
#undef GO
#undef RUN
  DS_CHECK_LAUNCH();
  return 0;
}

template <typename T>
int prepare(const void* proj, const float* conv_w, const float* conv_b, const void* conv_state, const float* a_log,
            const float* dt_bias, const int* seq_ids, const int* cu, const int* start, const int* slots, void* qk, void* v,
            float* gb, const ScanDims& D, hipStream_t st) {
  const int tile = D.T >= 512 ? TILE : 1;  // few tokens: as many waves as there are
  const bool vec = ((D.rows | D.q | D.k | D.v | D.dk | D.dv | D.conv | D.channels) & 3) == 0;
  const int cw = vec ? 256 : 64;
  const int64_t parts = 2 * ((D.Hk * D.dk + cw - 1) / cw) + (D.H * D.dv + cw - 1) / cw + (gb ? 1 : 0);
  const int64_t items = (D.T + tile - 1) / tile * parts;
  if (items > (int64_t)INT32_MAX * 4) return (int)hipErrorInvalidValue;
#define LAUNCH(TAPS, V)                                                                                               \
  hipLaunchKernelGGL((scan_prepare_kernel<T, TAPS, V>), dim3((unsigned)((items + 3) / 4)), dim3(256), 0, st, (const T*)proj, \
                     conv_w, conv_b, (const T*)conv_state, a_log, dt_bias, seq_ids, cu, start, slots, (T*)qk, (T*)v, gb,  \
                     tile, D)
  if (!vec) {
    if (D.taps == 1) LAUNCH(1, 1);
    else LAUNCH(0, 1);
  } else if (D.taps == 1) LAUNCH(1, 4);
  else if (D.taps == 2) LAUNCH(2, 4);
  else if (D.taps == 3) LAUNCH(3, 4);
  else if (D.taps == 4) LAUNCH(4, 4);
  else LAUNCH(0, 4);
#undef LAUNCH
  DS_CHECK_LAUNCH();
  return 0;
}

}  // namespace

// qk [2, Hk, T, dks] and v [H, T, dvs] in the storage type (padding must be zero before), gb [T, 2, H] fp32 (log decay,
// step size) or null for constant decays
extern "C" int ds_scan_prepare(const void* proj, const float* conv_w, const float* conv_b, const void* conv_state,
                               const float* a_log, const float* dt_bias, const int* seq_ids, const int* cu,
                               const int* start, const int* slots, void* qk, void* v, float* gb, const int* dims,
                               int tokens, int dtype, hipStream_t st) {
  if (tokens <= 0) return 0;
  const ScanDims D{dims[0], dims[1], dims[2], dims[3], dims[4], dims[5], dims[6], dims[7], dims[8], dims[9], dims[10], dims[11],
                   tokens};
  if (!scan_dims_ok(D) || (D.taps > 1 && (!conv_w || !conv_state)) || (gb && (!a_log || !dt_bias || D.dt < 0)))
    return (int)hipErrorInvalidValue;
  if (dtype == DS_F32)
    return prepare<float>(proj, conv_w, conv_b, conv_state, a_log, dt_bias, seq_ids, cu, start, slots, qk, v, gb, D, st);
  if (dtype == DS_BF16)
    return prepare<bf16>(proj, conv_w, conv_b, conv_state, a_log, dt_bias, seq_ids, cu, start, slots, qk, v, gb, D, st);
  return (int)hipErrorInvalidValue;
}

// The same tensors straight from the projection's columns (no convolution, no activation), the first 2 half columns of every
// head of q and k turned by cs [tokens, half, 2] (cos, sin). terms 2: qk [2, 2, Hk, T, dks] takes q and k as sums of two
extern "C" int ds_scan_split(const void* proj, const float* cs, int half, void* qk, void* v, int terms, const int* dims,
                             int tokens, int dtype, hipStream_t st) {
  if (tokens <= 0) return 0;
  const ScanDims D{dims[0], dims[1], dims[2], dims[3], dims[4], dims[5], dims[6], dims[7], dims[8], dims[9], dims[10], dims[11],
                   tokens};
  if (!scan_dims_ok(D) || half < 0 || 2 * half > D.dk || (half && !cs) || terms < 1 || terms > 2)
    return (int)hipErrorInvalidValue;
  const int64_t term = terms == 2 ? 2 * (int64_t)D.Hk * D.T * D.dks() : 0;
  const int all = D.rows | D.q | D.k | D.v | D.dk | D.dv | half;
#define GO(T, V) \
  hipLaunchKernelGGL((scan_split_kernel<T, V>), dim3(tokens), dim3(256), 0, st, (const T*)proj, cs, half, (T*)qk, (T*)v, term, D)
  if (dtype == DS_F32) {
    if (all % 4 == 0) GO(float, 4);
    else GO(float, 1);
  } else if (dtype == DS_BF16) {
    if (all % 8 == 0) GO(bf16, 8);
    else if (all % 4 == 0) GO(bf16, 4);
    else GO(bf16, 1);
  } else {
    return (int)hipErrorInvalidValue;
  }
#undef GO
  DS_CHECK_LAUNCH();
  return 0;
}

// list: sequences (indices into cu / start / slots) to run, `lstride` entries apart. zstate (null: no normaliser) [slots, H,
// ceil(dv / 32), dks] with floors [tokens, H]; terms: of q and k (ds_scan_split)
extern "C" int ds_scan_recur(const void* qk, const void* v, const float* gb, const float* log_decay, const float* skip,
                             float scale, const void* proj, float* state, float* zstate, const float* floors,
                             void* conv_state, int terms, const int* list, int nlist, int lstride,
                             const int* cu, const int* start, const int* slots, void* out, const int* dims, int tokens,
                             int dtype, hipStream_t st) {
  if (nlist <= 0) return 0;
  const ScanDims D{dims[0], dims[1], dims[2], dims[3], dims[4], dims[5], dims[6], dims[7], dims[8], dims[9], dims[10], dims[11],
                   tokens};
  if (!scan_dims_ok(D) || (!gb == !log_decay) || (!zstate != !floors) || terms < 1 || terms > 2 || (terms == 2 && zstate) ||
      (D.taps > 1 && !conv_state))
    return (int)hipErrorInvalidValue;
  if (dtype == DS_F32)
    return recur<float>(qk, v, gb, log_decay, skip, scale, proj, state, zstate, floors, conv_state, terms, list, nlist, lstride,
                        cu, start, slots, out, D, st);
  if (dtype == DS_BF16)
    return recur<bf16>(qk, v, gb, log_decay, skip, scale, proj, state, zstate, floors, conv_state, terms, list, nlist, lstride,
                       cu, start, slots, out, D, st);
  return (int)hipErrorInvalidValue;
}
