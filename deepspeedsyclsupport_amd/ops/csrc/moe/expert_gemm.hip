// Products of mixture-of-experts layers, CDNA4 (gfx950). A pair (token, choice) is entry t * K + k: inputs are read from row
// entry / div, results written to row `entry`, so nothing is copied into expert order and back. The gated form computes
// silu(gate) up of the same columns in one go; a plain product may end in a squared relu.
//
//  * stream: few rows per expert. bf16 weights are streamed once per tile of up to 64 entries. A workgroup owns 32 weight rows
//    of an expert (gated: 16 of the gate and the same 16 of the up part); its four waves take alternating 64-wide steps of the
//    inner dimension straight into registers: no LDS, no barrier until the sums meet.
//    The entries of an expert come from sorted lists or, for a few hundred of them, are picked out of the routing table by
//    every workgroup itself; then only the experts that occur get workgroups.
//  * tile: many rows per expert. 128 entries x 256 weight rows (gated: 128 of either part) per workgroup. Weights are stored in
//    operand order and every wave has rows of its own, so they go from memory to registers in 512-byte runs, one step of 64
//    ahead; only the entries' rows pass through LDS (swizzled, two buffers). Two workgroups share a CU. Workgroups walk groups
//    of 4 column tiles by all row tiles of an expert, so that those at work on an XCD at a time share both operands in its L2.
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
enum : int { NONE = 0, SILU_GLU = 1, RELU2 = 2 };  // activation codes
__device__ __forceinline__ float plain_act(float x, int act) {
  if (act != RELU2) return x;
  x = fmaxf(x, 0.f);
  return x * x;
}

struct ExpertArgs {
  const void* x;         // [.., K]
  const void* w;         // [E, N, K]; gated: [E, 2 N, K], gate rows first
  void* y;               // [entries, N]
  const int* experts;    // [entries]
  const int* offs;       // [E + 1] and
  const int* order;      // [entries], or null (up to FEW entries)
  int entries, E, N, K, div, act;
};

// Operand order of a weight matrix [rows, K] (ops/bf16_gemv.py): 16 x 64 tiles of 1024 elements, tile by tile along K;
// element [h][lane][j] of a tile is row lane % 16, column 16 (lane / 16) + 8 h + j

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

struct StreamShared {
  int list[FEW], words[MAXE / 32 + 1];
  f32x4 red[4][8][64];
};

// Entries m0 .. m0 + 16 MT - 1 of an expert, 32 weight rows (wp: this lane's row of either half)
template <int MT, bool GLU, bool SH>
__device__ __forceinline__ void stream_tile(const ExpertArgs& a, const bf16* const (&wp)[2], const int* ents, int cnt, int m0, int n0,
                                            StreamShared& sh) {
  const int lane = threadIdx.x & 63, l16 = lane & 15, q4 = lane >> 4, N = a.N, K = a.K;
  const int wid = __builtin_amdgcn_readfirstlane((int)threadIdx.x >> 6);
  const bf16* xp[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m)
    xp[m] = (const bf16*)a.x + (int64_t)(ents[min(m0 + 16 * m + l16, cnt - 1)] / a.div) * K + (SH ? 16 : 8) * q4;
  f32x4 acc[2][MT];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int m = 0; m < MT; ++m) acc[i][m] = f32x4{0.f, 0.f, 0.f, 0.f};
  // U steps of 64 of the inner dimension: all their loads, then the products
  auto steps = [&](auto count, int k0, bool tail) {
    constexpr int U = decltype(count)::value;
    bf16x8 wv[U][2][2], xv[U][2][MT];
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int c = 0; c < 2; ++c) {
          const int k = k0 + 256 * u + 32 * c, kc = tail ? min(k, K - 8 - 8 * q4) : k;
          const bf16* p = SH ? wp[i] + (int64_t)(k0 / 64 + 4 * u) * 1024 + 512 * c : wp[i] + kc;
          wv[u][c][i] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(p));
        }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int c = 0; c < 2; ++c) {
        const int k = k0 + 256 * u + (SH ? 8 : 32) * c, kc = tail ? min(k, K - 8 - 8 * q4) : k;
#pragma unroll
        for (int m = 0; m < MT; ++m) xv[u][c][m] = *reinterpret_cast<const bf16x8*>(xp[m] + kc);
        if (tail && k + 8 * q4 >= K) {  // columns past the width count as zero, on both sides
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
  constexpr int U = MT == 4 ? 2 : 4;
  const int whole = K / 64;
  int s = wid;
  for (; s + 4 * (U - 1) < whole; s += 4 * U) steps(Int<U>{}, 64 * s, false);
  for (; s < whole; s += 4) steps(Int<1>{}, 64 * s, false);
  if (!SH && K % 64 && whole % 4 == wid) steps(Int<1>{}, 64 * whole, true);
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int m = 0; m < MT; ++m) sh.red[wid][i * MT + m][lane] = acc[i][m];
  __syncthreads();
  auto total = [&](int j) {
    f32x4 s = sh.red[0][j][lane];
#pragma unroll
    for (int v = 1; v < 4; ++v) s += sh.red[v][j][lane];
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
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] = plain_act(v[i], a.act);
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

template <bool GLU, bool SH>
__global__ void __launch_bounds__(256) expert_stream_kernel(ExpertArgs a) {
  __shared__ StreamShared sh;
  const int lane = threadIdx.x & 63, l16 = lane & 15, q4 = lane >> 4;
  int e = blockIdx.y, cnt;
  const int* ents = sh.list;
  if (a.offs) {
    cnt = a.offs[e + 1] - a.offs[e];
    ents = a.order + a.offs[e];
  } else {
    cnt = collect(a, blockIdx.y, sh.list, sh.words, e);
  }
  const int N = a.N, n0 = blockIdx.x * (GLU ? 16 : 32);
  if (cnt == 0) return;
  const bf16* w = (const bf16*)a.w + (int64_t)e * (GLU ? 2 : 1) * N * a.K;
  const bf16* wp[2];
  if constexpr (SH) {  // (16 divides N)
    wp[0] = w + (int64_t)n0 * a.K + lane * 8;
    wp[1] = GLU ? wp[0] + (int64_t)N * a.K : w + (int64_t)min(n0 + 16, N - 16) * a.K + lane * 8;
  } else {
    wp[0] = w + (int64_t)min(n0 + l16, N - 1) * a.K + 8 * q4;
    wp[1] = GLU ? wp[0] + (int64_t)N * a.K : w + (int64_t)min(n0 + 16 + l16, N - 1) * a.K + 8 * q4;
  }
  for (int m0 = 0; m0 < cnt;) {  // (uniform over the workgroup) as narrow as the rest allows
    const int left = cnt - m0;
    if (left <= 16) stream_tile<1, GLU, SH>(a, wp, ents, cnt, m0, n0, sh);
    else if (left <= 32) stream_tile<2, GLU, SH>(a, wp, ents, cnt, m0, n0, sh);
    else stream_tile<4, GLU, SH>(a, wp, ents, cnt, m0, n0, sh);
    m0 += left <= 16 ? 16 : left <= 32 ? 32 : 64;
  }
}

// ------------------------------------------------------------------------------------------------ many rows per expert
constexpr int BM = 128, BN = 256, GROUP = 4;

template <bool GLU>
__global__ void __launch_bounds__(256, 2) expert_tile_kernel(ExpertArgs a) {
  __shared__ __attribute__((aligned(16))) bf16 xs[2][BM * 64];
  __shared__ int pre[MAXE + 1], offs[MAXE + 1], ents[BM], found;
  const int tid = threadIdx.x, lane = tid & 63, l32 = lane & 31, hh = lane >> 5;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int N = a.N, K = a.K, KQ = K / 64, per = GLU ? BN / 2 : BN, nt = (N + per - 1) / per;
  // ---- row tiles of all experts laid end to end; this workgroup's place among them
  for (int i = tid; i <= a.E; i += 256) offs[i] = a.offs[i];
  __syncthreads();
  if (tid < 64) {
    int c[4], s = 0;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int e = 4 * lane + i;
      c[i] = e < a.E ? (offs[e + 1] - offs[e] + BM - 1) / BM : 0;
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
      if (4 * lane + i < a.E) pre[4 * lane + i] = at;
      at += c[i];
    }
    if (lane == 63) pre[a.E] = run;
  }
  __syncthreads();
  const int total = pre[a.E] * nt;
  if ((int)blockIdx.x >= total) return;
  const int id = xcd_remap(blockIdx.x, total);
  for (int e = tid; e < a.E; e += 256)
    if (pre[e] * nt <= id && id < pre[e + 1] * nt) found = e;
  __syncthreads();
  const int e = found, mt = pre[e + 1] - pre[e], local = id - pre[e] * nt, g = local / (mt * GROUP);
  const int rest = local - g * mt * GROUP, width = min(GROUP, nt - g * GROUP);
  const int m0 = rest / width * BM, n0 = (g * GROUP + rest % width) * per;
  const int left = min(BM, offs[e + 1] - offs[e] - m0);
  if (tid < BM) ents[tid] = a.order[offs[e] + m0 + min(tid, left - 1)];
  __syncthreads();
  // ---- entries' rows on their way to LDS: 8 rows of 8 pieces per wave and access, piece p of row r holding columns
  // 8 (p ^ (r / 2 % 8)) .. + 7
  const bf16* xp[4];
  int xo[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = wid * 32 + i * 8 + (lane >> 3), p = lane & 7;
    xp[i] = (const bf16*)a.x + (int64_t)(ents[r] / a.div) * K + 8 * (p ^ ((r >> 1) & 7));
    xo[i] = r * 64 + p * 8;
  }
  // ---- this wave's 2 x 32 weight rows: gate and up of the same columns, or 64 neighbours
  const bf16* wp[2];
#pragma unroll
  for (int t = 0; t < 2; ++t) {
    const int row = GLU ? min(n0 + wid * 32, N - 32) + t * N : min(n0 + wid * 64 + 32 * t, N - 32);
    wp[t] = (const bf16*)a.w + ((int64_t)e * (GLU ? 2 : 1) * N + row + (l32 & 16)) * K + (hh * 16 + (l32 & 15)) * 8;
  }
  bf16x8 xr[4], wa[2][2][2], wb[2][2][2];  // [t][h][j]: columns 16 (2 j + hh) + 8 h .. + 7 of the step
  f32x16 acc[2][4];
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[t][m][r] = 0.f;
  auto load_x = [&](int kq) {
#pragma unroll
    for (int i = 0; i < 4; ++i) xr[i] = *reinterpret_cast<const bf16x8*>(xp[i] + kq * 64);
  };
  auto load_w = [&](bf16x8 (&w)[2][2][2], int kq) {
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int h = 0; h < 2; ++h)
#pragma unroll
        for (int j = 0; j < 2; ++j)
          w[t][h][j] = *reinterpret_cast<const bf16x8*>(wp[t] + (int64_t)kq * 1024 + h * 512 + j * 256);
  };
  auto store_x = [&](int buf) {
#pragma unroll
    for (int i = 0; i < 4; ++i) *reinterpret_cast<bf16x8*>(&xs[buf][xo[i]]) = xr[i];
  };
  const int tiles = (left + 31) / 32, sw = (l32 >> 1) & 7;
  auto compute = [&](const bf16x8 (&w)[2][2][2], int buf) {
#pragma unroll
    for (int h = 0; h < 2; ++h)
#pragma unroll
      for (int j = 0; j < 2; ++j)
#pragma unroll
        for (int m = 0; m < 4; ++m) {
          if (m >= tiles) break;  // (the branch also keeps the operands of later steps out of the registers)
          const bf16x8 x = *reinterpret_cast<const bf16x8*>(&xs[buf][(32 * m + l32) * 64 + 8 * ((4 * j + 2 * hh + h) ^ sw)]);
#pragma unroll
          for (int t = 0; t < 2; ++t) acc[t][m] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(w[t][h][j], x, acc[t][m], 0, 0, 0);
        }
  };
  load_w(wa, 0);
  load_x(0);
  store_x(0);
  __syncthreads();
  for (int kq = 0; kq < KQ; kq += 2) {
    if (kq + 1 < KQ) {
      load_x(kq + 1);
      load_w(wb, kq + 1);
    }
    compute(wa, 0);
    if (kq + 1 >= KQ) break;
    store_x(1);
    __syncthreads();
    if (kq + 2 < KQ) {
      load_x(kq + 2);
      load_w(wa, kq + 2);
    }
    compute(wb, 1);
    if (kq + 2 < KQ) store_x(0);
    __syncthreads();
  }
  // lane: entry l32 of a tile, weight rows 8 q + 4 hh + 0..3
#pragma unroll
  for (int m = 0; m < 4; ++m) {
    const int r = 32 * m + l32;
    if (r >= left) continue;
    bf16* yr = (bf16*)a.y + (int64_t)ents[r] * N;
#pragma unroll
    for (int t = 0; t < (GLU ? 1 : 2); ++t) {
      const int n = GLU ? n0 + wid * 32 : n0 + wid * 64 + 32 * t;
      if (n >= N) continue;
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        bf16x4 o;
#pragma unroll
        for (int i = 0; i < 4; ++i)
          o[i] = (bf16)(GLU ? silu_mul(acc[0][m][4 * q + i], acc[1][m][4 * q + i]) : plain_act(acc[t][m][4 * q + i], a.act));
        *reinterpret_cast<bf16x4*>(yr + n + 8 * q + 4 * hh) = o;
      }
    }
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
    else s = plain_act(s, a.act);
    if (lane == 0) ((T*)a.y)[i * a.N + n] = (T)s;
  }
}

// out[t] = sum_k w[t, k] y[row(t, k)] (+ base[t])
template <typename T>
__global__ void __launch_bounds__(256) expert_sum_kernel(const T* __restrict__ y, const float* __restrict__ w,
                                                         const int* __restrict__ rows, const T* __restrict__ base,
                                                         T* __restrict__ out, int W, int K) {
  const int64_t t = blockIdx.x;
  for (int c = threadIdx.x; c < W; c += 256) {
    float v = 0.f;
    for (int k = 0; k < K; ++k) v = fmaf(w[t * K + k], (float)y[(rows ? rows[t * K + k] : t * K + k) * W + c], v);
    out[t * W + c] = (T)(base ? v + (float)base[t * W + c] : v);
  }
}

}  // namespace

extern "C" int ds_expert_few() { return FEW; }
extern "C" int ds_expert_order_ok(int N, int K) { return N % 32 == 0 && K % 64 == 0; }

// y[i] = w[experts[i]] x[i / div] for every entry; act SILU_GLU: silu of the first N rows times the others; RELU2: max(., 0)^2. offs and order from
// ds_expert_place, or null for up to ds_expert_few() entries. operand: the weights are in operand order (N % 32, K % 64 must
// be 0); then with lists and `tile` the many-rows kernel runs.
extern "C" int ds_expert_gemm(const void* x, const void* w, void* y, const int* experts, const int* offs, const int* order,
                              int entries, int E, int N, int K, int div, int act, int operand, int tile, int dtype,
                              hipStream_t st) {
  if (entries <= 0) return 0;
  if (E <= 0 || E > MAXE || N <= 0 || K <= 0 || div <= 0 || (!offs != !order) || (N + 63) / 64 > 65535)
    return (int)hipErrorInvalidValue;
  const bool lists = offs != nullptr, gated = act == SILU_GLU;
  if (operand && (dtype != DS_BF16 || !ds_expert_order_ok(N, K) || (!lists && entries > FEW))) return (int)hipErrorInvalidValue;
  const ExpertArgs a{x, w, y, experts, offs, order, entries, E, N, K, div, act};
  if (operand && lists && tile) {
    const int per = gated ? BN / 2 : BN;
    const int64_t grid = ((int64_t)entries / BM + E) * ((N + per - 1) / per);
    if (grid > INT32_MAX) return (int)hipErrorInvalidValue;
    if (gated) hipLaunchKernelGGL(expert_tile_kernel<true>, dim3((unsigned)grid), dim3(256), 0, st, a);
    else hipLaunchKernelGGL(expert_tile_kernel<false>, dim3((unsigned)grid), dim3(256), 0, st, a);
    DS_CHECK_LAUNCH();
    return 0;
  }
  if (operand || (dtype == DS_BF16 && K % 8 == 0 && (lists || entries <= FEW))) {
    const dim3 grid((N + (gated ? 15 : 31)) / (gated ? 16 : 32), lists ? E : (entries < E ? entries : E));
#define GO(SH)                                                                                              \
  {                                                                                                         \
    if (gated) hipLaunchKernelGGL((expert_stream_kernel<true, SH>), grid, dim3(256), 0, st, a);             \
    else hipLaunchKernelGGL((expert_stream_kernel<false, SH>), grid, dim3(256), 0, st, a);                  \
  }
    if (operand) GO(true)
    else GO(false)
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

extern "C" int ds_expert_sum(const void* y, const float* w, const int* rows, const void* base, void* out, int T, int W, int K, int dtype,
                             hipStream_t st) {
  if (T <= 0) return 0;
  if (W <= 0 || K <= 0) return (int)hipErrorInvalidValue;
  if (dtype == DS_F32)
    hipLaunchKernelGGL(expert_sum_kernel<float>, dim3(T), dim3(256), 0, st, (const float*)y, w, rows,
                       (const float*)base, (float*)out, W, K);
  else if (dtype == DS_BF16)
    hipLaunchKernelGGL(expert_sum_kernel<bf16>, dim3(T), dim3(256), 0, st, (const bf16*)y, w, rows,
                       (const bf16*)base, (bf16*)out, W, K);
  else return (int)hipErrorInvalidValue;
  DS_CHECK_LAUNCH();
  return 0;
}
