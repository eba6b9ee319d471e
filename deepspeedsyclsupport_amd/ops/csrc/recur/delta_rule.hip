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
//  * prepare: one wave per (token, head part): convolution + silu + unit norm / decays, reading earlier tokens of the
//    same portion from the projection itself and the ones before it from the sequence's state slot. Everything that
//    enters the recurrence leaves it in fp32 (v in the storage type: it is a convolution output).
//  * recur: one workgroup per (sequence, head); the state sits in registers (LPC lanes per value column, E rows each)
//    while the portion's tokens pass one by one: decoding and short portions. It also moves the convolution's window
//    on in the state slot (prepare, which reads the old one, has finished by then).
// A sequence whose portion starts at position 0 starts from zero: slots need no clearing between owners.
#include "delta_rule.h"

namespace {

template <typename T>
__global__ void __launch_bounds__(256) delta_prepare_kernel(
    const T* __restrict__ proj, const float* __restrict__ conv_w, const T* __restrict__ conv_state,
    const float* __restrict__ a_log, const float* __restrict__ dt_bias, const int* __restrict__ seq_ids,
    const int* __restrict__ cu, const int* __restrict__ start, const int* __restrict__ slots, float* __restrict__ qk,
    T* __restrict__ v_out, float* __restrict__ gb, int tokens, DeltaDims D) {
  const int parts = 2 * D.Hk + D.H + 1, lane = threadIdx.x & 63;
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= (int64_t)tokens * parts) return;
  const int t = (int)(item / parts), part = (int)(item % parts);
  const int NP = D.row(), C = D.channels();
  if (part == parts - 1) {  // decays (as logarithms) and write strengths
    const T* b = proj + (int64_t)t * NP + C + D.H * D.dv;
    for (int h = lane; h < D.H; h += 64) {
      const float z = (float)b[D.H + h] + dt_bias[h];
      const float sp = z > 20.f ? z : log1pf(expf(z));
      gb[((int64_t)t * 2) * D.H + h] = -expf(a_log[h]) * sp;
      gb[((int64_t)t * 2 + 1) * D.H + h] = 1.f / (1.f + expf(-(float)b[h]));
    }
    return;
  }
  const bool is_v = part >= 2 * D.Hk;
  const int width = is_v ? D.dv : D.dk;
  const int c0 = is_v ? 2 * D.Hk * D.dk + (part - 2 * D.Hk) * D.dv : part * D.dk;
  const int seq = seq_ids[t], j = t - cu[seq];  // index of the token in its portion
  const bool fresh = start[seq] == 0;
  const T* cs = conv_state + (int64_t)slots[seq] * (D.taps - 1) * C;
  auto conv = [&](int c) {
    float a = 0.f;
    for (int i = 0; i < D.taps; ++i) {
      const int src = j - (D.taps - 1) + i;  // relative to the portion's first token
      float x = 0.f;
      if (src >= 0) x = (float)proj[(int64_t)(t - j + src) * NP + c];
      else if (!fresh) x = (float)cs[(int64_t)(src + D.taps - 1) * C + c];
      a = fmaf(conv_w[(int64_t)c * D.taps + i], x, a);
    }
    return silu(a);
  };
  if (is_v) {
    T* dst = v_out + (int64_t)t * D.H * D.dv + (part - 2 * D.Hk) * D.dv;
    for (int c = lane; c < width; c += 64) dst[c] = (T)conv(c0 + c);
    return;
  }
  float vals[4], ss = 0.f;  // dk <= 256
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int c = i * 64 + lane;
    vals[i] = c < width ? conv(c0 + c) : 0.f;
    ss = fmaf(vals[i], vals[i], ss);
  }
  float r = 1.f / sqrtf(wave_sum(ss) + 1e-6f);
  if (part < D.Hk) r *= 1.f / sqrtf((float)D.dk);
  float* dst = qk + (int64_t)t * 2 * D.Hk * D.dk + (int64_t)part * D.dk;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int c = i * 64 + lane;
    if (c < width) dst[c] = vals[i] * r;
  }
}

template <typename T, int E>
__global__ void __launch_bounds__(1024) delta_recur_kernel(
    const float* __restrict__ qk, const T* __restrict__ v, const float* __restrict__ gb, const T* __restrict__ proj,
    const float* __restrict__ norm_w, float eps, float* __restrict__ state, T* __restrict__ conv_state,
    const int* __restrict__ list, const int* __restrict__ cu, const int* __restrict__ start,
    const int* __restrict__ slots, T* __restrict__ out, DeltaDims D, int lpc) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int seq = list[blockIdx.x], h = blockIdx.y, hk = h / (D.H / D.Hk), tid = threadIdx.x;
  const int kp = lpc * E;  // padded key width
  float* qs = sm;
  float* ks = sm + kp;
  float* red = sm + 2 * kp;
  const int64_t t0 = cu[seq];
  const int n = cu[seq + 1] - (int)t0;
  const bool fresh = start[seq] == 0;
  const int NP = D.row(), C = D.channels(), col = tid / lpc, p = tid % lpc;
  const bool on = col < D.dv;
  float* st = state + ((int64_t)slots[seq] * D.H + h) * D.dk * D.dv;
  float S[E];
#pragma unroll
  for (int i = 0; i < E; ++i) {
    const int k = p + lpc * i;
    S[i] = (on && !fresh && k < D.dk) ? st[(int64_t)k * D.dv + col] : 0.f;
  }
  for (int t = 0; t < n; ++t) {
    const int64_t tok = t0 + t;
    const float* qr = qk + (tok * 2 * D.Hk + hk) * D.dk;
    const float* kr = qr + (int64_t)D.Hk * D.dk;
    __syncthreads();
    for (int c = tid; c < kp; c += blockDim.x) {
      qs[c] = c < D.dk ? qr[c] : 0.f;
      ks[c] = c < D.dk ? kr[c] : 0.f;
    }
    const float g = expf(gb[tok * 2 * D.H + h]), beta = gb[(tok * 2 + 1) * D.H + h];
    const float vv = on ? (float)v[(tok * D.H + h) * D.dv + col] : 0.f;
    __syncthreads();
    float a = 0.f;
#pragma unroll
    for (int i = 0; i < E; ++i) {
      S[i] *= g;
      a = fmaf(S[i], ks[p + lpc * i], a);
    }
    for (int o = 1; o < lpc; o <<= 1) a += __shfl_xor(a, o, 64);
    const float u = beta * (vv - a);
    float ov = 0.f;
#pragma unroll
    for (int i = 0; i < E; ++i) {
      S[i] = fmaf(ks[p + lpc * i], u, S[i]);
      ov = fmaf(S[i], qs[p + lpc * i], ov);
    }
    for (int o = 1; o < lpc; o <<= 1) ov += __shfl_xor(ov, o, 64);
    const float ss = block_sum(on && p == 0 ? ov * ov : 0.f, red);
    const float rs = 1.f / sqrtf(ss / (float)D.dv + eps);
    if (on && p == 0) {
      const float gate = (float)proj[tok * NP + C + h * D.dv + col];
      out[(tok * D.H + h) * D.dv + col] = (T)(ov * rs * norm_w[col] * silu(gate));
    }
  }
  if (on) {
#pragma unroll
    for (int i = 0; i < E; ++i) {
      const int k = p + lpc * i;
      if (k < D.dk) st[(int64_t)k * D.dv + col] = S[i];
    }
  }
  if (D.taps > 1) advance_head(conv_state + (int64_t)slots[seq] * (D.taps - 1) * C, proj, t0, n, D, fresh, h);
}

template <typename T>
int recur(const float* qk, const void* v, const float* gb, const void* proj, const float* norm_w, float eps, float* state,
          void* conv_state, const int* list, int nlist, const int* cu, const int* start, const int* slots, void* out,
          DeltaDims D, hipStream_t st) {
  int lpc = 1;
  while (lpc < 16 && ((D.dk + lpc - 1) / lpc > 32 || lpc * D.dv < 128) && lpc * 2 * D.dv <= 1024) lpc *= 2;
  const int e = (D.dk + lpc - 1) / lpc, nt = (lpc * D.dv + 63) / 64 * 64;
#define GO(E)                                                                                                       \
  hipLaunchKernelGGL((delta_recur_kernel<T, E>), dim3(nlist, D.H), dim3(nt), (size_t)(2 * lpc * E + 16) * 4, st, qk,  \
                     (const T*)v, gb, (const T*)proj, norm_w, eps, state, (T*)conv_state, list, cu, start, slots,     \
                     (T*)out, D, lpc)
  if (e <= 4) GO(4);
  else if (e <= 8) GO(8);
  else if (e <= 16) GO(16);
  else if (e <= 32) GO(32);
  else if (e <= 64) GO(64);
  else return (int)hipErrorInvalidValue;
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
  const DeltaDims D{Hk, H, dk, dv, taps};
  if (!dims_ok(D)) return (int)hipErrorInvalidValue;
  const int64_t items = (int64_t)tokens * (2 * Hk + H + 1);
#define GO(T)                                                                                                       \
  hipLaunchKernelGGL((delta_prepare_kernel<T>), dim3((unsigned)((items + 3) / 4)), dim3(256), 0, st, (const T*)proj,  \
                     conv_w, (const T*)conv_state, a_log, dt_bias, seq_ids, cu, start, slots, qk, (T*)v, gb, tokens, D)
  if (dtype == DS_F32) GO(float);
  else if (dtype == DS_BF16) GO(bf16);
  else return (int)hipErrorInvalidValue;
#undef GO
  DS_CHECK_LAUNCH();
  return 0;
}

// list: the sequences (indices into cu / start / slots) to run
extern "C" int ds_delta_recur(const float* qk, const void* v, const float* gb, const void* proj, const float* norm_w,
                              float eps, float* state, void* conv_state, const int* list, int nlist, const int* cu,
                              const int* start, const int* slots, void* out, int Hk, int H, int dk, int dv, int taps,
                              int dtype, hipStream_t st) {
  if (nlist <= 0) return 0;
  const DeltaDims D{Hk, H, dk, dv, taps};
  if (!dims_ok(D)) return (int)hipErrorInvalidValue;
  if (dtype == DS_F32)
    return recur<float>(qk, v, gb, proj, norm_w, eps, state, conv_state, list, nlist, cu, start, slots, out, D, st);
  if (dtype == DS_BF16)
    return recur<bf16>(qk, v, gb, proj, norm_w, eps, state, conv_state, list, nlist, cu, start, slots, out, D, st);
  return (int)hipErrorInvalidValue;
}
