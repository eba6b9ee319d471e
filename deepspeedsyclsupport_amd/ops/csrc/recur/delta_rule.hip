// Gated delta rule with short causal convolutions (linear attention with a carried state), CDNA4 (gfx950).
//
// Per head, with a state S [dk, dv] in fp32 that starts at zero:
//     S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
// k and q are unit vectors per head (q scaled by dk^-1/2) made from projections that passed a causal convolution over
// the sequence's last `taps` tokens and silu; g = exp(-exp(A_log) softplus(a + dt_bias)), beta = sigmoid(b). Each head's
// o is RMS-normalised over dv, scaled by a shared weight and gated by silu of a projection.
//
// The fused projection row of a token is [q (Hk dk) | k (Hk dk) | v (H dv) | g (H dv) | b (H) | a (H)].
//
//  * prepare: one wave per (few consecutive tokens, head part): convolution + silu + unit norm / decays, reading earlier tokens of the
//    same portion from the projection itself and the ones before it from the sequence's state slot. Everything that
//    enters the recurrence leaves it in fp32 (v in the storage type: it is a convolution output).
//  * recur: one workgroup per (sequence, head); the state, kept as [dv, dk] (dk padded to 4), sits in registers
//    while the portion's tokens pass one by one: decoding and short portions. It also moves the convolution's window
//    on in the state slot (prepare, which reads the old one, has finished by then).
// A sequence whose portion starts at position 0 starts from zero: slots need no clearing between owners.
#include "delta_rule.h"

namespace {

constexpr int TILE = 8;  // consecutive tokens a prepare wave walks

// TAPS: filter length, the tile's inputs in registers; 0: any length, inputs read per tap. PAIR: even head sizes.
template <typename T, int TAPS, bool PAIR>
__global__ void __launch_bounds__(256) delta_prepare_kernel(
    const T* __restrict__ proj, const float* __restrict__ conv_w, const T* __restrict__ conv_state,
    const float* __restrict__ a_log, const float* __restrict__ dt_bias, const int* __restrict__ seq_ids,
    const int* __restrict__ cu, const int* __restrict__ start, const int* __restrict__ slots, float* __restrict__ qk,
    T* __restrict__ v_out, float* __restrict__ gb, int tokens, int tile, DeltaDims D) {
  const int parts = 2 * D.Hk + D.H + 1, lane = threadIdx.x & 63;
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  const int t_lo = (int)(item / parts) * tile, part = (int)(item % parts), t_hi = min(t_lo + tile, tokens);
  if (t_lo >= tokens) return;
  const int NP = D.row(), CH = D.channels(), taps = TAPS ? TAPS : D.taps;
  if (part == parts - 1) {  // decays (as logarithms) and write strengths
    for (int t = t_lo; t < t_hi; ++t) {
      const T* b = proj + (int64_t)t * NP + CH + D.H * D.dv;
      for (int h = lane; h < D.H; h += 64) {
        const float z = (float)b[D.H + h] + dt_bias[h];
        const float sp = z > 20.f ? z : log1pf(expf(z));
        gb[((int64_t)t * 2) * D.H + h] = -expf(a_log[h]) * sp;
        gb[((int64_t)t * 2 + 1) * D.H + h] = 1.f / (1.f + expf(-(float)b[h]));
      }
    }
    return;
  }
  const bool is_v = part >= 2 * D.Hk;
  const int width = is_v ? D.dv : D.dk;
  const int c0 = is_v ? 2 * D.Hk * D.dk + (part - 2 * D.Hk) * D.dv : part * D.dk;
  for (int ta = t_lo; ta < t_hi;) {  // runs of tokens of one sequence
    const int seq = seq_ids[ta], first = cu[seq], tb = min(t_hi, cu[seq + 1]), n = tb - ta, j0 = ta - first;
    const T* cs = start[seq] == 0 ? nullptr : conv_state + (int64_t)slots[seq] * (taps - 1) * CH;
    // the convolution's input row at place j of the portion (negative: before it); zero tells that there is none
    auto row = [&](int j, float& zero) {
      zero = j >= 0 || cs ? 1.f : 0.f;
      return j >= 0 || !cs ? proj + (int64_t)(first + max(j, 0)) * NP + c0 : cs + (int64_t)(j + taps - 1) * CH + c0;
    };
    float y[TILE][2][2];
#pragma unroll
    for (int k = 0; k < 2; ++k) {  // a lane's channels: 2 lane, 2 lane + 1, and the same 128 further on
      const int c = k * 128 + 2 * lane;
      if (k * 128 >= width) {
#pragma unroll
        for (int t = 0; t < TILE; ++t) y[t][k][0] = y[t][k][1] = 0.f;
      } else if constexpr (TAPS != 0) {
        float x[TILE + TAPS - 1][2], cw[2][TAPS];
#pragma unroll
        for (int i = 0; i < TILE + TAPS - 1; ++i) {
          float zero;
          const T* r = row(j0 + min(i, n + TAPS - 2) - (TAPS - 1), zero);
          load2<PAIR>(r, c, width, x[i]);
          x[i][0] *= zero;
          x[i][1] *= zero;
        }
#pragma unroll
        for (int e = 0; e < 2; ++e)
#pragma unroll
          for (int i = 0; i < TAPS; ++i)
            cw[e][i] = conv_w[(int64_t)(c0 + min(c + e, width - 1)) * TAPS + i] * (c + e < width ? 1.f : 0.f);
#pragma unroll
        for (int t = 0; t < TILE; ++t)
#pragma unroll
          for (int e = 0; e < 2; ++e) {
            float acc = 0.f;
#pragma unroll
            for (int i = 0; i < TAPS; ++i) acc = fmaf(cw[e][i], x[t + i][e], acc);
            y[t][k][e] = silu(acc);  // 0 beyond the width
          }
      } else {
        float acc[TILE][2];
#pragma unroll
        for (int t = 0; t < TILE; ++t) acc[t][0] = acc[t][1] = 0.f;
        for (int i = 0; i < taps; ++i) {
          const float w0 = c < width ? conv_w[(int64_t)(c0 + c) * taps + i] : 0.f;
          const float w1 = c + 1 < width ? conv_w[(int64_t)(c0 + c + 1) * taps + i] : 0.f;
#pragma unroll
          for (int t = 0; t < TILE; ++t) {
            float zero, x[2];
            const T* r = row(j0 + min(t, n - 1) - (taps - 1) + i, zero);
            load2<PAIR>(r, c, width, x);
            acc[t][0] = fmaf(w0, x[0] * zero, acc[t][0]);
            acc[t][1] = fmaf(w1, x[1] * zero, acc[t][1]);
          }
        }
#pragma unroll
        for (int t = 0; t < TILE; ++t) {
          y[t][k][0] = silu(acc[t][0]);
          y[t][k][1] = silu(acc[t][1]);
        }
      }
    }
#pragma unroll
    for (int t = 0; t < TILE; ++t) {
      if (t >= n) break;
      const int64_t tok = ta + t;
      if (is_v) {
#pragma unroll
        for (int k = 0; k < 2; ++k)
          store2<PAIR>(v_out + D.v_at(part - 2 * D.Hk, tok), k * 128 + 2 * lane, width, y[t][k]);
        continue;
      }
      float ss = 0.f;
#pragma unroll
      for (int k = 0; k < 2; ++k) ss = fmaf(y[t][k][0], y[t][k][0], fmaf(y[t][k][1], y[t][k][1], ss));
      float r = 1.f / sqrtf(wave_sum(ss) + 1e-6f);
      if (part < D.Hk) r *= 1.f / sqrtf((float)D.dk);
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        y[t][k][0] *= r;
        y[t][k][1] *= r;
        store2<true>(qk + D.q_at(part, tok), k * 128 + 2 * lane, D.dks(), y[t][k]);
      }
    }
    ta = tb;
  }
}

// LPC lanes per value column, each with 4 NV key rows in quads: row 4 (p + LPC i) + e. The state is stored with the key
// index innermost, [dv, dk], so a column's lanes read consecutive 16-byte pieces.
template <typename T, int NV, int LPC>
__global__ void __launch_bounds__(1024) delta_recur_kernel(
    const float* __restrict__ qk, const T* __restrict__ v, const float* __restrict__ gb, const T* __restrict__ proj,
    const float* __restrict__ norm_w, float eps, float* __restrict__ state, T* __restrict__ conv_state,
    const int* __restrict__ list, const int* __restrict__ cu, const int* __restrict__ start,
    const int* __restrict__ slots, T* __restrict__ out, DeltaDims D) {
  constexpr int KP = 4 * NV * LPC;  // padded key width
  __shared__ __attribute__((aligned(16))) float qs[KP];
  __shared__ __attribute__((aligned(16))) float ks[KP];
  __shared__ float red[16];
  const int seq = list[blockIdx.x], h = blockIdx.y, hk = h / (D.H / D.Hk), tid = threadIdx.x;
  const int64_t t0 = cu[seq];
  const int n = cu[seq + 1] - (int)t0;
  const bool fresh = start[seq] == 0;
  const int NP = D.row(), C = D.channels(), col = tid / LPC, p = tid % LPC;
  const bool on = col < D.dv;
  float* st = state + (((int64_t)slots[seq] * D.H + h) * D.dv + col) * D.dks();
  f32x4 S[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int k = 4 * (p + LPC * i);
    S[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (on && !fresh && k < D.dk) S[i] = *reinterpret_cast<const f32x4*>(st + k);
  }
  for (int t = 0; t < n; ++t) {
    const int64_t tok = t0 + t;
    const float* qr = qk + D.q_at(hk, tok);
    const float* kr = qk + D.k_at(hk, tok);
    __syncthreads();
    for (int c = tid; c < KP; c += blockDim.x) {
      qs[c] = c < D.dk ? qr[c] : 0.f;
      ks[c] = c < D.dk ? kr[c] : 0.f;
    }
    const float g = expf(gb[tok * 2 * D.H + h]), beta = gb[(tok * 2 + 1) * D.H + h];
    const float vv = on ? (float)v[D.v_at(h, tok) + col] : 0.f;
    __syncthreads();
    float a = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const f32x4 k4 = *reinterpret_cast<const f32x4*>(ks + 4 * (p + LPC * i));
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[i][e] *= g;
        a = fmaf(S[i][e], k4[e], a);
      }
    }
#pragma unroll
    for (int o = 1; o < LPC; o <<= 1) a += __shfl_xor(a, o, 64);
    const float u = beta * (vv - a);
    float ov = 0.f;
    asm volatile("" ::: "memory");  // keys come from LDS again: holding them costs the occupancy
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const f32x4 k4 = *reinterpret_cast<const f32x4*>(ks + 4 * (p + LPC * i));
      const f32x4 q4 = *reinterpret_cast<const f32x4*>(qs + 4 * (p + LPC * i));
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[i][e] = fmaf(k4[e], u, S[i][e]);
        ov = fmaf(S[i][e], q4[e], ov);
      }
    }
#pragma unroll
    for (int o = 1; o < LPC; o <<= 1) ov += __shfl_xor(ov, o, 64);
    const float ss = block_sum(on && p == 0 ? ov * ov : 0.f, red);
    const float rs = 1.f / sqrtf(ss / (float)D.dv + eps);
    if (on && p == 0) {
      const float gate = (float)proj[tok * NP + C + h * D.dv + col];
      out[(tok * D.H + h) * D.dv + col] = (T)(ov * rs * norm_w[col] * silu(gate));
    }
  }
  if (on) {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int k = 4 * (p + LPC * i);
      if (k < D.dk) *reinterpret_cast<f32x4*>(st + k) = S[i];
    }
  }
  if (D.taps > 1) advance_head(conv_state + (int64_t)slots[seq] * (D.taps - 1) * C, proj, t0, n, D, fresh, h);
}

template <typename T>
int recur(const float* qk, const void* v, const float* gb, const void* proj, const float* norm_w, float eps, float* state,
          void* conv_state, const int* list, int nlist, const int* cu, const int* start, const int* slots, void* out,
          DeltaDims D, hipStream_t st) {
  // 8 lanes per column where the workgroup allows it (128-byte pieces of the state per column), fewer for wide heads
  const int q = (D.dk + 3) / 4, lpc = D.dv <= 128 ? 8 : 4, nt = (lpc * D.dv + 63) / 64 * 64, nv = (q + lpc - 1) / lpc;
#define GO(NV, LPC)                                                                                                  \
  hipLaunchKernelGGL((delta_recur_kernel<T, NV, LPC>), dim3(nlist, D.H), dim3(nt), 0, st, qk, (const T*)v, gb,         \
                     (const T*)proj, norm_w, eps, state, (T*)conv_state, list, cu, start, slots, (T*)out, D)
#define ROW(LPC)             \
  {                          \
    if (nv <= 1) GO(1, LPC); \
    else if (nv <= 2) GO(2, LPC); \
    else if (nv <= 4) GO(4, LPC); \
    else if (nv <= 8) GO(8, LPC); \
    else GO(16, LPC);        \
  }
  if (lpc == 8) ROW(8)
  else ROW(4)
#undef ROW
#undef GO
  DS_CHECK_LAUNCH();
  return 0;
}

}  // namespace

extern "C" int ds_delta_prepare(const void* proj, const float* conv_w, const void* conv_state, const float* a_log,
                                const float* dt_bias, const int* seq_ids, const int* cu, const int* start,
                                const int* slots, float* qk, void* v, float* gb, int tokens, int Hk, int H, int dk,
                                int dv, int taps, int dtype, hipStream_t st) {
  if (tokens <= 0) return 0;
  const DeltaDims D{Hk, H, dk, dv, taps, tokens};
  if (!dims_ok(D)) return (int)hipErrorInvalidValue;
  const int tile = tokens >= 512 ? TILE : 1;  // few tokens: as many waves as there are
  const int64_t items = (int64_t)((tokens + tile - 1) / tile) * (2 * Hk + H + 1);
  const bool pair = dk % 2 == 0 && dv % 2 == 0;
#define LAUNCH(T, TAPS, PAIR)                                                                                       \
  hipLaunchKernelGGL((delta_prepare_kernel<T, TAPS, PAIR>), dim3((unsigned)((items + 3) / 4)), dim3(256), 0, st,      \
                     (const T*)proj, conv_w, (const T*)conv_state, a_log, dt_bias, seq_ids, cu, start, slots, qk, (T*)v, gb, \
                     tokens, tile, D)
#define GO(T)                                  \
  {                                            \
    if (!pair) LAUNCH(T, 0, false);            \
    else if (taps == 4) LAUNCH(T, 4, true);    \
    else if (taps == 3) LAUNCH(T, 3, true);    \
    else if (taps == 2) LAUNCH(T, 2, true);    \
    else LAUNCH(T, 0, true);                   \
  }
  if (dtype == DS_F32) GO(float)
  else if (dtype == DS_BF16) GO(bf16)
  else return (int)hipErrorInvalidValue;
#undef GO
#undef LAUNCH
  DS_CHECK_LAUNCH();
  return 0;
}

// list: the sequences (indices into cu / start / slots) to run
extern "C" int ds_delta_recur(const float* qk, const void* v, const float* gb, const void* proj, const float* norm_w,
                              float eps, float* state, void* conv_state, const int* list, int nlist, const int* cu,
                              const int* start, const int* slots, void* out, int tokens, int Hk, int H, int dk, int dv,
                              int taps, int dtype, hipStream_t st) {
  if (nlist <= 0) return 0;
  const DeltaDims D{Hk, H, dk, dv, taps, tokens};
  if (!dims_ok(D)) return (int)hipErrorInvalidValue;
  if (dtype == DS_F32)
    return recur<float>(qk, v, gb, proj, norm_w, eps, state, conv_state, list, nlist, cu, start, slots, out, D, st);
  if (dtype == DS_BF16)
    return recur<bf16>(qk, v, gb, proj, norm_w, eps, state, conv_state, list, nlist, cu, start, slots, out, D, st);
  return (int)hipErrorInvalidValue;
}
