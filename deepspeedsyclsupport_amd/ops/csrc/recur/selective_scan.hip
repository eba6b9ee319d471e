// Selective scan: recurrences with a decay of their own per channel and state, CDNA4 (gfx950).
//
// Every channel c carries N numbers in fp32 that start at zero. With step = softplus(dt + dt_bias) and given A[c, n] < 0:
//     S[c, n] <- exp(step_c A[c, n]) S[c, n] + step_c x_c B_n;   y_c = sum_n S[c, n] C_n + D_c x_c;   out_c = y_c silu(z_c)
// B and C belong to the token, shared by all channels. There is one exponential and four multiplications per number and token
// and nothing for the matrix cores to do: long portions are bound by the vector unit and by LDS reads, decoding by the state.
//
//  * scan (long portions): a workgroup of four waves takes 256 / LP neighbouring channels of one sequence and walks its new
//    tokens, TT at a time. LP lanes share a channel, NPL numbers each, in registers throughout. LP is chosen so that a SIMD gets
//    two waves at least (a single one issues at little more than half the rate): few lanes per channel spend the least on what
//    a channel does once per token, many make a single long sequence parallel.
//      stage: step and step * x of every (token, channel) of the tile, B and C, all fp32, into LDS; x and z stay with the thread
//        that will write the same (token, channel). The next tile's operands are on their way meanwhile.
//      walk: token by token without barriers, LDS rows along the tokens, so that a read brings two of them. Shares of y of LP
//        tokens meet in the lanes whose tokens they are: pairs of lanes trade halves, log2 LP times.
//      write: y from LDS, skip and gate applied, in whole rows.
//  * step (decodes, short portions): four numbers per lane, nothing but registers, so that many waves stream the states.
//
// The channels' convolution windows move on as well, but for portions of one token, where the convolution has done it. A
// sequence whose portion starts at position 0 starts from zero: slots need no clearing between owners.
#include "ds_hip.h"

#include <type_traits>

namespace {

constexpr int NT = 256;
constexpr float LOG2E = 1.4426950408889634f;

struct SelArgs {
  const void *x, *dt, *bc, *z, *cx;       // x, dt [T, C]; bc [T, B | C]; z, cx [T, C]: columns, rows ld* apart
  int64_t ldbc, ldz, ldcx;
  const float *dt_bias, *decay, *skip;    // [C], [C, N], [C]
  float* state;                           // [slots, C, NS]
  void* conv;                             // [slots, taps - 1, C]: last rows of cx, or null
  const int *list, *cu, *start, *slots;   // list: sequences, `stride` apart
  void* out;                              // [T, C]
  int C, N, NS, taps, seqs, stride;
};

__device__ __forceinline__ float exp_f(float v) { return __builtin_amdgcn_exp2f(v * LOG2E); }
// log(1 + e^v) to a few units in the last place: what adding 1 rounds off is put right by the last factor
__device__ __forceinline__ float softplus_f(float v) {
  constexpr float LN2 = 0.6931471805599453f;
  const float u = exp_f(-fabsf(v)), w = 1.f + u, d = w - 1.f;
  return fmaxf(v, 0.f) + (d == 0.f ? u : __builtin_amdgcn_logf(w) * (LN2 * u * __builtin_amdgcn_rcpf(d)));
}
__device__ __forceinline__ float silu_f(float z) { return z * __builtin_amdgcn_rcpf(1.f + exp_f(-z)); }

// V neighbouring elements
template <typename T, int V>
struct Few {
  typedef T TV __attribute__((ext_vector_type(2)));
  T v[V];
  __device__ __forceinline__ void load(const T* p) {
    if constexpr (V == 2) *reinterpret_cast<TV*>(v) = *reinterpret_cast<const TV*>(p);
    else v[0] = p[0];
  }
};
template <typename T, int V>
__device__ __forceinline__ void store_few(T* p, const float (&f)[V]) {
  typedef T TV __attribute__((ext_vector_type(2)));
  if constexpr (V == 2) *reinterpret_cast<TV*>(p) = TV{(T)f[0], (T)f[1]};
  else p[0] = (T)f[0];
}

template <int CTRL>
__device__ __forceinline__ float dpp(float v) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}
constexpr int XOR1 = 0xb1, XOR2 = 0x4e, MIRROR8 = 0x141, MIRROR16 = 0x140;  // lane moves within 4, 8, 16

// p[i]: this lane's share of a sum for token i of LP. Returns the sum over the group of LP lanes of the shares of the lane's own
// token: in every step pairs of lanes trade halves of what they hold.
template <int LP>
__device__ __forceinline__ float trade(float (&p)[LP], int g) {
  auto step = [&](auto move, int n) {
    const bool up = g & n;
#pragma unroll
    for (int i = 0; i < n; ++i) {
      const float keep = up ? p[n + i] : p[i], give = up ? p[i] : p[n + i];
      p[i] = keep + dpp<decltype(move)::value>(give);
    }
  };
  if constexpr (LP == 16) step(std::integral_constant<int, MIRROR16>{}, 8);
  if constexpr (LP >= 8) step(std::integral_constant<int, MIRROR8>{}, 4);
  step(std::integral_constant<int, XOR2>{}, 2);
  step(std::integral_constant<int, XOR1>{}, 1);
  return p[0];
}

// A channel's convolution window: the last taps - 1 of [old window | the portion's inputs]
template <typename T>
__device__ __forceinline__ void advance_window(const SelArgs& a, int64_t slot, int t0, int n, bool old, int c) {
  constexpr int FEW = 4;
  const int w = a.taps - 1;
  T* cs = (T*)a.conv + slot * w * a.C + c;
  auto at = [&](int j) {  // place j of the new window
    const int src = n + j;
    if (src >= w) return ((const T*)a.cx)[(int64_t)(t0 + src - w) * a.ldcx + c];
    return old ? cs[(int64_t)src * a.C] : (T)0.f;
  };
  if (w <= FEW) {  // all loads, then all stores
    T v[FEW];
#pragma unroll
    for (int j = 0; j < FEW; ++j)
      if (j < w) v[j] = at(j);
#pragma unroll
    for (int j = 0; j < FEW; ++j)
      if (j < w) cs[(int64_t)j * a.C] = v[j];
  } else {
    for (int j = 0; j < w; ++j) cs[(int64_t)j * a.C] = at(j);  // ascending: src > j, so nothing is overwritten before it is read
  }
}

// V: channels a thread stages and writes
template <typename T, int LP, int NPL, int V>
__global__ void __launch_bounds__(NT) selective_scan_kernel(SelArgs a) {
  constexpr int CH = NT / LP, NW = LP * NPL;               // channels; numbers per channel as they are laid out in LDS
  constexpr int TT = LP == 4 || NW > 128 ? 16 : 32;        // tokens of a tile
  constexpr int CV = CH / V, PR = NT / CV;                 // threads across the channels, tokens they stage at a time
  constexpr int PER = (TT + PR - 1) / PR;
  constexpr int U = NPL >= 8 ? 2 : LP / 2 < 4 ? LP / 2 : 4;  // tokens whose operands are read ahead
  constexpr int ROW = TT + 2;                              // tokens of an LDS row: an odd number of 16-byte pieces
  constexpr int LANE = NPL * ROW + (NPL % 2 ? 0 : 2);      // a lane's rows of B and C: also odd, so that lanes use all banks
  __shared__ __attribute__((aligned(16))) f32x2 sx[CH + 1][ROW];  // step, step * x (reads ahead run over the end)
  __shared__ __attribute__((aligned(16))) f32x2 sb[LP * LANE + ROW];  // B, C
  __shared__ float sy[TT][CH];
  const int blocks = (a.C + CH - 1) / CH, id = xcd_remap(blockIdx.x, gridDim.x);
  const int seq = a.list[id / blocks * a.stride], c0 = id % blocks * CH, tid = threadIdx.x;
  const int t0 = a.cu[seq], n = a.cu[seq + 1] - t0;
  const int64_t slot = a.slots[seq];
  if (n <= 0) return;
  const bool old = a.start[seq] > 0;
  // ---- this lane's numbers
  const int g = tid % LP, cl = tid / LP, c = min(c0 + cl, a.C - 1), n0 = g * NPL;
  const bool mine = c0 + cl < a.C;
  float* st = a.state + (slot * a.C + c) * a.NS + n0;
  float S[NPL], A[NPL];
#pragma unroll
  for (int i = 0; i < NPL; ++i) {
    A[i] = 0.f;
    S[i] = 0.f;
    if (n0 + i < a.N) {
      A[i] = a.decay[(int64_t)c * a.N + n0 + i] * LOG2E;
      if (old) S[i] = st[i];
    }
  }
  // ---- what this thread stages and writes: tokens wt + PR j, channels wc .. wc + V - 1
  const int wl = tid % CV * V, wt = tid / CV, wc = c0 + wl, wcc = min(wc, a.C - V);
  const bool on = wc < a.C;
  float bias[V], skip[V];
#pragma unroll
  for (int v = 0; v < V; ++v) {
    bias[v] = a.dt_bias[wcc + v];
    skip[v] = a.skip[wcc + v];
  }
  constexpr int BPER = (TT * NW + NT - 1) / NT;
  const T *xp = (const T*)a.x + (int64_t)t0 * a.C + wcc, *dp = (const T*)a.dt + (int64_t)t0 * a.C + wcc;
  const T *zp = (const T*)a.z + t0 * a.ldz + wcc, *bp = (const T*)a.bc + t0 * a.ldbc;
  int xo[PER], zo[PER], bo[BPER];  // places of a whole tile's operands
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    xo[j] = (wt + PR * j) * a.C;
    zo[j] = (wt + PR * j) * (int)a.ldz;
  }
#pragma unroll
  for (int j = 0; j < BPER; ++j) {
    const int e = tid + NT * j;
    bo[j] = min(e / NW, TT - 1) * (int)a.ldbc + min(e % NW, a.N - 1);
  }
  Few<T, V> xr[PER], dr[PER], zr[PER];
  T br[BPER], cr[BPER];
  auto fetch = [&](int k0) {
    const int last = n - 1 - k0;
    const T *x = xp + (int64_t)k0 * a.C, *d = dp + (int64_t)k0 * a.C, *z = zp + k0 * a.ldz, *b = bp + k0 * a.ldbc;
    if (last >= PR * PER - 1 && last >= TT - 1) {
#pragma unroll
      for (int j = 0; j < PER; ++j) {
        xr[j].load(x + xo[j]);
        dr[j].load(d + xo[j]);
        zr[j].load(z + zo[j]);
      }
#pragma unroll
      for (int j = 0; j < BPER; ++j) {
        br[j] = b[bo[j]];
        cr[j] = b[bo[j] + a.N];
      }
    } else {  // rows past the end repeat the last one
#pragma unroll
      for (int j = 0; j < PER; ++j) {
        const int r = min(wt + PR * j, last);
        xr[j].load(x + r * a.C);
        dr[j].load(d + r * a.C);
        zr[j].load(z + r * a.ldz);
      }
#pragma unroll
      for (int j = 0; j < BPER; ++j) {
        const int e = tid + NT * j;
        const T* q = b + min(e / NW, last) * a.ldbc + min(e % NW, a.N - 1);
        br[j] = q[0];
        cr[j] = q[a.N];
      }
    }
  };
  struct Ahead {  // two tokens at a time
    f32x4 sd[U / 2], b[U / 2][NPL];
  };
  auto read = [&](Ahead& r, int t) {
#pragma unroll
    for (int u = 0; u < U / 2; ++u) {
      r.sd[u] = *reinterpret_cast<const f32x4*>(&sx[cl][t + 2 * u]);
#pragma unroll
      for (int i = 0; i < NPL; ++i) r.b[u][i] = *reinterpret_cast<const f32x4*>(&sb[g * LANE + i * ROW + t + 2 * u]);
    }
  };
  fetch(0);
  for (int k0 = 0; k0 < n; k0 += TT) {
    const int m = min(TT, n - k0);
    float xs[PER][V], gate[PER][V];
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int r = wt + PR * j;
      f32x2 sd[V];
#pragma unroll
      for (int v = 0; v < V; ++v) {
        xs[j][v] = (float)xr[j].v[v];
        gate[j][v] = silu_f((float)zr[j].v[v]);
        float step = softplus_f((float)dr[j].v[v] + bias[v]);
        step = r < m ? step : 0.f;  // steps of zero leave the numbers as they are
        sd[v] = f32x2{step, step * xs[j][v]};
      }
      if (TT % PR && r >= TT) continue;
#pragma unroll
      for (int v = 0; v < V; ++v) sx[wl + v][r] = sd[v];
    }
#pragma unroll
    for (int j = 0; j < BPER; ++j) {
      const int e = tid + NT * j;
      const int i = e % NW;
      if ((TT * NW) % NT == 0 || e < TT * NW)
        sb[i / NPL * LANE + i % NPL * ROW + e / NW] = i < a.N ? f32x2{(float)br[j], (float)cr[j]} : f32x2{0.f, 0.f};
    }
    __syncthreads();
    if (k0 + TT < n) fetch(k0 + TT);
    Ahead r[2];
    read(r[0], 0);
#pragma unroll 1
    for (int t = 0; t < m; t += LP) {  // rounds of LP tokens
      float p[LP];
#pragma unroll
      for (int w = 0; w < LP / U; ++w) {
        read(r[(w + 1) % 2], t + (w + 1) * U);
        const Ahead& now = r[w % 2];
        float e[U][NPL];
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
          for (int k = 0; k < NPL; ++k) e[u][k] = __builtin_amdgcn_exp2f(now.sd[u / 2][u % 2 * 2] * A[k]);
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const float dx = now.sd[u / 2][u % 2 * 2 + 1];
          float sum = 0.f;
#pragma unroll
          for (int k = 0; k < NPL; ++k) {
            S[k] = fmaf(e[u][k], S[k], dx * now.b[u / 2][k][u % 2 * 2]);
            const float cn = now.b[u / 2][k][u % 2 * 2 + 1];
            sum = k ? fmaf(S[k], cn, sum) : S[k] * cn;
          }
          p[w * U + u] = sum;
        }
      }
      sy[t + g][cl] = trade<LP>(p, g);
    }
    __syncthreads();
    T* out = (T*)a.out + (int64_t)(t0 + k0) * a.C + wcc;
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int r = wt + PR * j;
      if (r >= m || !on) continue;
      float y[V];
#pragma unroll
      for (int v = 0; v < V; ++v) y[v] = fmaf(skip[v], xs[j][v], sy[r][wl + v]) * gate[j][v];
      store_few<T, V>(out + xo[j], y);
    }
  }
  if (mine) {
#pragma unroll
    for (int i = 0; i < NPL; ++i)
      if (n0 + i < a.N) st[i] = S[i];
  }
  if (a.conv && n > 1 && tid < CH && c0 + tid < a.C) advance_window<T>(a, slot, t0, n, old, c0 + tid);
}

// Four numbers per lane, LP lanes per channel, R sequences at a time. VEC: N is 4 LP, and B and C lie in 4-element pieces
template <typename T, int LP, bool VEC, int R>
__global__ void __launch_bounds__(NT) selective_step_kernel(SelArgs a) {
  typedef T T4 __attribute__((ext_vector_type(4)));
  constexpr int CH = NT / LP;
  const int tid = threadIdx.x, g = tid % LP, n0 = 4 * g, cw = (int)blockIdx.x * CH + tid / LP, c = min(cw, a.C - 1);
  const bool mine = cw < a.C;
  int t0[R], n[R], longest = 0;
  bool old[R];
  int64_t slot[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int i = (int)blockIdx.y * R + r, seq = a.list[min(i, a.seqs - 1) * a.stride];
    t0[r] = a.cu[seq];
    n[r] = i < a.seqs ? a.cu[seq + 1] - t0[r] : 0;
    old[r] = a.start[seq] > 0;
    slot[r] = a.slots[seq];
    longest = max(longest, n[r]);
  }
  auto place = [&](int r) { return a.state + (slot[r] * a.C + c) * a.NS + n0; };
  f32x4 S[R], A = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int r = 0; r < R; ++r) {
    S[r] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (!old[r]) continue;
    if constexpr (VEC) {
      S[r] = *reinterpret_cast<const f32x4*>(place(r));
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (n0 + i < a.N) S[r][i] = place(r)[i];
    }
  }
  if constexpr (VEC) {
    A = *reinterpret_cast<const f32x4*>(a.decay + (int64_t)c * a.N + n0);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n0 + i < a.N) A[i] = a.decay[(int64_t)c * a.N + n0 + i];
  }
  A *= LOG2E;
  const float bias = a.dt_bias[c], skip = a.skip[c];
  for (int k = 0; k < longest; ++k) {
    float x[R], z[R], step[R];
    f32x4 B[R], C[R];
#pragma unroll
    for (int r = 0; r < R; ++r) {  // (a sequence that is through repeats its last token's operands)
      const int64_t t = max(t0[r] + min(k, n[r] - 1), 0);
      x[r] = (float)((const T*)a.x)[t * a.C + c];
      z[r] = (float)((const T*)a.z)[t * a.ldz + c];
      step[r] = (float)((const T*)a.dt)[t * a.C + c];
      const T* b = (const T*)a.bc + t * a.ldbc + n0;
      B[r] = f32x4{0.f, 0.f, 0.f, 0.f};
      C[r] = B[r];
      if constexpr (VEC) {
        const T4 b4 = *reinterpret_cast<const T4*>(b), c4 = *reinterpret_cast<const T4*>(b + a.N);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          B[r][i] = (float)b4[i];
          C[r][i] = (float)c4[i];
        }
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (n0 + i < a.N) {
            B[r][i] = (float)b[i];
            C[r][i] = (float)b[a.N + i];
          }
      }
    }
#pragma unroll
    for (int r = 0; r < R; ++r) {
      if (k >= n[r]) continue;
      const float s = softplus_f(step[r] + bias), dx = s * x[r];
      float y = 0.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        S[r][i] = fmaf(__builtin_amdgcn_exp2f(s * A[i]), S[r][i], dx * B[r][i]);
        y = fmaf(S[r][i], C[r][i], y);
      }
#pragma unroll
      for (int o = LP / 2; o > 0; o >>= 1) y += __shfl_xor(y, o, 64);
      if (g == 0 && mine) ((T*)a.out)[(int64_t)(t0[r] + k) * a.C + c] = (T)(fmaf(skip, x[r], y) * silu_f(z[r]));
    }
  }
  if (!mine) return;
#pragma unroll
  for (int r = 0; r < R; ++r) {
    if (n[r] <= 0) continue;
    if constexpr (VEC) {
      *reinterpret_cast<f32x4*>(place(r)) = S[r];
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (n0 + i < a.N) place(r)[i] = S[r][i];
    }
    if (a.conv && n[r] > 1 && g == 0) advance_window<T>(a, slot[r], t0[r], n[r], old[r], c);
  }
}

template <typename T, int LP, int V>
int launch(const SelArgs& a, hipStream_t st) {
  constexpr int CH = NT / LP;
  const int64_t grid = (int64_t)((a.C + CH - 1) / CH) * a.seqs;
  if (grid > INT32_MAX) return (int)hipErrorInvalidValue;
  const int need = (a.N + LP - 1) / LP;
#define GO(NPL)                                                                                                    \
  {                                                                                                                \
    hipLaunchKernelGGL((selective_scan_kernel<T, LP, NPL, V>), dim3((unsigned)grid), dim3(NT), 0, st, a);          \
    DS_CHECK_LAUNCH();                                                                                             \
    return 0;                                                                                                      \
  }
  if (need <= 1) GO(1)
  if (need <= 2) GO(2)
  if (need <= 4) GO(4)
  if constexpr (LP < 16) {
    if (need <= 6) GO(6)
  }
  if (need <= 8) GO(8)
  if constexpr (LP == 16) {
    if (need <= 16) GO(16)
  }
#undef GO
  return (int)hipErrorInvalidValue;
}

template <typename T, int V>
int scan(const SelArgs& a, hipStream_t st) {
  // as few lanes per channel as give the chip's 1024 SIMDs work (a second wave each is worth more than fewer lanes)
  const int64_t waves = (int64_t)a.C * a.seqs / 16;  // with 4
  if (a.N <= 32 && waves >= 1536) return launch<T, 4, V>(a, st);
  if (a.N <= 64 && waves >= 512) return launch<T, 8, V>(a, st);
  return launch<T, 16, V>(a, st);
}

template <typename T>
int step(const SelArgs& a, bool aligned, hipStream_t st) {
  const int need = (a.N + 3) / 4;
#define RUN(LP, VEC, R)                                                                                                  \
  hipLaunchKernelGGL((selective_step_kernel<T, LP, VEC, R>), dim3((a.C + NT / LP - 1) / (NT / LP), (a.seqs + R - 1) / R), \
                     dim3(NT), 0, st, a)
#define GO(LP)                                                                                    \
  if (need <= LP) {                                                                               \
    if (aligned && a.N == 4 * LP) {                                                               \
      if ((int64_t)a.C * a.seqs * LP >= (int64_t)2048 * NT) RUN(LP, true, 4);                     \
      else RUN(LP, true, 1);                                                                      \
    } else {                                                                                      \
      RUN(LP, false, 1);                                                                          \
    }                                                                                             \
    DS_CHECK_LAUNCH();                                                                            \
    return 0;                                                                                     \
  }
  GO(1) GO(2) GO(4) GO(8) GO(16) GO(32) GO(64)
#undef GO
#undef RUN
  return (int)hipErrorInvalidValue;
}

}  // namespace

// Numbers per channel a kernel instance holds
extern "C" int ds_selective_scan_max() { return 256; }

// Sequences list[0], list[stride], ... (`seqs` of them). x, dt [T, C] and, ldbc / ldz / ldcx elements from row to row,
// bc [T, B | C (N each)], z [T, C], cx [T, C]; state [slots, C, NS]; conv [slots, taps - 1, C] or null. `steps`: few tokens each
extern "C" int ds_selective_scan(const void* x, const void* dt, const void* bc, int64_t ldbc, const void* z, int64_t ldz,
                                 const float* dt_bias, const float* decay, const float* skip, float* state, const void* cx,
                                 int64_t ldcx, void* conv, const int* list, int seqs, int stride, const int* cu, const int* start,
                                 const int* slots, void* out, int steps, int C, int N, int NS, int taps, int dtype,
                                 hipStream_t st) {
  if (seqs <= 0) return 0;
  if (C <= 0 || N <= 0 || N > ds_selective_scan_max() || NS < N || taps < 1 || (conv && (taps < 2 || !cx)) || stride <= 0 ||
      seqs > 65535)
    return (int)hipErrorInvalidValue;
  // (places within a tile are 32-bit)
  if (((int64_t)C + ldz + ldbc) * 64 > INT32_MAX) return (int)hipErrorInvalidValue;
  const SelArgs a{x,    dt,   bc,   z,   cx,    ldbc,  ldz, ldcx, dt_bias, decay, skip, state,
                  conv, list, cu, start, slots, out, C,   N,    NS,      taps,  seqs, stride};
  const int el = dtype == DS_F32 ? 4 : 2;
  if (steps) {
    const bool aligned = NS % 4 == 0 && ldbc % 4 == 0 && N % 4 == 0 && ((uintptr_t)bc & (4 * el - 1)) == 0 &&
                         (((uintptr_t)state | (uintptr_t)decay) & 15) == 0;
    if (dtype == DS_F32) return step<float>(a, aligned, st);
    if (dtype == DS_BF16) return step<bf16>(a, aligned, st);
    return (int)hipErrorInvalidValue;
  }
  const bool two = C % 2 == 0 && ldz % 2 == 0 && (((uintptr_t)x | (uintptr_t)dt | (uintptr_t)z) & 3) == 0;
  if (dtype == DS_F32) return scan<float, 1>(a, st);
  if (dtype == DS_BF16) return two ? scan<bf16, 2>(a, st) : scan<bf16, 1>(a, st);
  return (int)hipErrorInvalidValue;
}
