// Attention over paged latents for decodes and short portions, bf16, CDNA4 (gfx950). See latent_ops.hip for the layout.
//
// With the key map folded into the query, all heads share one key row per token, [latent (R) | rotated part (r)], and its
// first R columns are the value: a cached byte is read once for every head of every new token of a sequence. The (token,
// head) pairs of a sequence are rows of one matrix; a workgroup takes 16 MR of them and a range of keys (split so that the
// launch covers the chip), 64 keys at a time:
//  * the key tile sits in LDS (the next one is on its way in registers), the queries too;
//  * scores: wave w takes keys 16 w .. 16 w + 15, K Q^T on the matrix cores, so a lane has one row's scores;
//  * softmax weights go through LDS as two bf16 terms (16 mantissa bits);
//  * values: O^T += V^T P^T, wave w a quarter of the latent's columns; V^T comes out of the same key tile by transposing
//    LDS reads.
// Ranges leave fp32 partial sums that a combine pass merges. The sink, if there is one, joins the denominator once, at the end.
// With a sliding window the ranges start where the sequence's first new token sees its first key.
#include "ds_hip.h"

namespace {

constexpr int NT = 256;
constexpr int BN = 64;
constexpr int PP = BN + 8;  // LDS row of the weights
constexpr float LOG2E = 1.4426950408889634f;

typedef short s16x4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ f32x4 mfma(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

struct LatArgs {
  const bf16* q;     // [T, H, R + r], the key map folded in
  const bf16* lat;   // [blocks, BS, R + r]
  bf16* out;         // [T, H, R]
  float* acc;        // [splits, T H, R] partial sums, unnormalised
  float* ml;         // [splits, T H, 2] maximum (log2 units) and sum
  const int* bt;
  const int* cu;
  const int* start;
  const float* sink;  // [H] or null
  int first, tok_base, H, R, r, BS, max_blocks, range, splits, window;
  int64_t rows;  // T H
  float c;       // scale * log2(e)
};

// NV: 16-column value tiles per wave (R <= 64 NV); NP: 16-byte pieces of a key row in steps of 4 (R + r <= 32 NP)
template <int MR, int NV>
__global__ void __launch_bounds__(NT) latent_decode_kernel(LatArgs a) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int W = a.R + a.r, WP = (W + 31) & ~31, KP = WP + 8, rows_b = 16 * MR;
  bf16* const Ks = reinterpret_cast<bf16*>(smem);       // [BN][KP] (value tiles past the row's end read what follows)
  bf16* const Qs = Ks + BN * KP;                        // [16 MR][KP]
  bf16* const Ps = Qs + rows_b * KP;                    // [2][16 MR][PP]
  float* const red = reinterpret_cast<float*>(Ps + 2 * rows_b * PP);  // [4][16 MR]
  const int s = a.first + blockIdx.x, split = blockIdx.z, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int l16 = lane & 15, q4 = lane >> 4;
  const int tok0 = a.cu[s] - a.tok_base, n = a.cu[s + 1] - a.cu[s], nrow = n * a.H, row0 = blockIdx.y * rows_b;
  if (row0 >= nrow) return;
  const int st = a.start[s];
  // keys this block may see: up to the last row's position
  const int end = st + min(n - 1, (row0 + rows_b - 1) / a.H) + 1;
  const int k_lo = (a.window > 0 ? max(st - a.window + 1, 0) : 0) + split * a.range, k_hi = min(end, k_lo + a.range);
  const int64_t g0 = (int64_t)tok0 * a.H + row0;  // first row in q / out
  if (k_lo >= k_hi) {  // nothing in this range: the combine pass must not read what was never written
    if (a.splits > 1 && tid < rows_b && row0 + tid < nrow) {
      float* ml = a.ml + ((int64_t)split * a.rows + g0 + tid) * 2;
      ml[0] = -INFINITY;
      ml[1] = 0.f;
    }
    return;
  }
  const int* bt = a.bt + (int64_t)s * a.max_blocks;
  const int CPR = WP / 8, pieces = W / 8;  // 16-byte pieces per LDS row, and those that exist
  bf16x8 zero8;
#pragma unroll
  for (int e = 0; e < 8; ++e) zero8[e] = (bf16)0.f;
  for (int i = tid; i < rows_b * CPR; i += NT) {
    const int row = i / CPR, ch = i % CPR;
    *reinterpret_cast<bf16x8*>(Qs + row * KP + ch * 8) =
        ch < pieces ? *reinterpret_cast<const bf16x8*>(a.q + (g0 + min(row, nrow - 1 - row0)) * W + ch * 8) : zero8;
  }
  // Key rows in flight: a row's pieces belong to 4 neighbouring threads, piece (tid & 3) + 4 i
  constexpr int NP = NV == 1 ? 4 : NV == 2 ? 6 : NV == 4 ? 10 : 18;
  bf16x8 kr[NP];
  const int krow = tid >> 2, kch = tid & 3;
  auto fetch = [&](int k0) {
    const int key = min(k0 + krow, k_hi - 1);
    const bf16* src = a.lat + ((int64_t)bt[key / a.BS] * a.BS + key % a.BS) * W;
#pragma unroll
    for (int i = 0; i < NP; ++i) kr[i] = *reinterpret_cast<const bf16x8*>(src + min(kch + 4 * i, pieces - 1) * 8);
  };
  auto stage = [&]() {
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      const int ch = kch + 4 * i;
      if (ch < CPR) *reinterpret_cast<bf16x8*>(Ks + krow * KP + ch * 8) = ch < pieces ? kr[i] : zero8;
    }
  };
  int pos[MR], lo[MR];  // position of this lane's row in every row tile, and the first key it sees
#pragma unroll
  for (int m = 0; m < MR; ++m) {
    pos[m] = st + min(row0 + 16 * m + l16, nrow - 1) / a.H;
    lo[m] = a.window > 0 ? pos[m] - a.window + 1 : 0;
  }
  f32x4 o[MR][NV];
  float m_run[MR], l_run[MR];
#pragma unroll
  for (int m = 0; m < MR; ++m) {
    m_run[m] = -INFINITY;
    l_run[m] = 0.f;
#pragma unroll
    for (int t = 0; t < NV; ++t) o[m][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  fetch(k_lo);
  for (int k0 = k_lo; k0 < k_hi; k0 += BN) {
    stage();
    if (k0 + BN < k_hi) fetch(k0 + BN);
    lds_barrier();
    f32x4 sc[MR];
#pragma unroll
    for (int m = 0; m < MR; ++m) sc[m] = f32x4{0.f, 0.f, 0.f, 0.f};
    const bf16* kp = Ks + (16 * w + l16) * KP + 8 * q4;
    const bf16* qp = Qs + l16 * KP + 8 * q4;
    for (int k = 0; k < WP; k += 32) {
      const bf16x8 kf = *reinterpret_cast<const bf16x8*>(kp + k);
#pragma unroll
      for (int m = 0; m < MR; ++m) sc[m] = mfma(kf, *reinterpret_cast<const bf16x8*>(qp + 16 * m * KP + k), sc[m]);
    }
    // lane: row l16 of tile m, keys 16 w + 4 q4 + 0..3
#pragma unroll
    for (int m = 0; m < MR; ++m) {
      float mx = -INFINITY;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int key = k0 + 16 * w + 4 * q4 + j;
        sc[m][j] = key <= pos[m] && key < k_hi && key >= lo[m] ? sc[m][j] * a.c : -INFINITY;
        mx = fmaxf(mx, sc[m][j]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      if (q4 == 0) red[w * rows_b + 16 * m + l16] = mx;
    }
    lds_barrier();
#pragma unroll
    for (int m = 0; m < MR; ++m) {
      float mx = m_run[m];
#pragma unroll
      for (int v = 0; v < 4; ++v) mx = fmaxf(mx, red[v * rows_b + 16 * m + l16]);
      const float use = mx == -INFINITY ? 0.f : mx;
      const float alpha = exp2f(m_run[m] - use);  // (nothing in sight yet: 0, of sums that are 0)
      m_run[m] = mx;
      bf16x4 hi, rest;
      float sum = 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float p = exp2f(sc[m][j] - use);
        sum += p;
        hi[j] = (bf16)p;
        rest[j] = (bf16)(p - (float)hi[j]);
      }
      l_run[m] = l_run[m] * alpha + sum;
      *reinterpret_cast<bf16x4*>(Ps + (16 * m + l16) * PP + 16 * w + 4 * q4) = hi;
      *reinterpret_cast<bf16x4*>(Ps + (rows_b + 16 * m + l16) * PP + 16 * w + 4 * q4) = rest;
      if (!__all(alpha == 1.f)) {
#pragma unroll
        for (int t = 0; t < NV; ++t) o[m][t] *= alpha;
      }
    }
    lds_barrier();
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      bf16x8 ph[MR], pl[MR];
#pragma unroll
      for (int m = 0; m < MR; ++m) {
        const bf16* p = Ps + (16 * m + l16) * PP + 32 * ks + 8 * q4;
        ph[m] = *reinterpret_cast<const bf16x8*>(p);
        pl[m] = *reinterpret_cast<const bf16x8*>(p + rows_b * PP);
      }
#pragma unroll
      for (int t = 0; t < NV; ++t) {
        const bf16* b = Ks + (32 * ks + 8 * q4 + (l16 >> 2)) * KP + (w * NV + t) * 16 + 4 * (l16 & 3);
        const s16x4_t x = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4_t*)b);
        const s16x4_t y = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4_t*)(b + 4 * KP));
        s16x8 vv;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          vv[e] = x[e];
          vv[4 + e] = y[e];
        }
        const bf16x8 vf = __builtin_bit_cast(bf16x8, vv);
#pragma unroll
        for (int m = 0; m < MR; ++m) {
          o[m][t] = mfma(vf, pl[m], o[m][t]);
          o[m][t] = mfma(vf, ph[m], o[m][t]);
        }
      }
    }
    lds_barrier();
  }
  // sums of the rows over the waves' keys
#pragma unroll
  for (int m = 0; m < MR; ++m) {
    float l = l_run[m];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (q4 == 0) red[w * rows_b + 16 * m + l16] = l;
  }
  lds_barrier();
#pragma unroll
  for (int m = 0; m < MR; ++m) {
    const int row = row0 + 16 * m + l16;
    if (row >= nrow) continue;
    float l = 0.f;
#pragma unroll
    for (int v = 0; v < 4; ++v) l += red[v * rows_b + 16 * m + l16];
    const int64_t gr = g0 + 16 * m + l16;
    if (a.splits == 1) {
      float mx = m_run[m], f = 1.f;
      if (a.sink) {
        const float sk = a.sink[row % a.H] * LOG2E, mn = fmaxf(mx, sk);
        f = exp2f(mx - mn);
        l = l * f + exp2f(sk - mn);
      }
      f /= l;
#pragma unroll
      for (int t = 0; t < NV; ++t) {
        const int cv = (w * NV + t) * 16 + 4 * q4;
        bf16x4 v;
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = (bf16)(o[m][t][j] * f);
        if (cv < a.R) *reinterpret_cast<bf16x4*>(a.out + gr * a.R + cv) = v;
      }
    } else {
      const int64_t pr = (int64_t)split * a.rows + gr;
#pragma unroll
      for (int t = 0; t < NV; ++t) {
        const int cv = (w * NV + t) * 16 + 4 * q4;
        if (cv < a.R) *reinterpret_cast<f32x4*>(a.acc + pr * a.R + cv) = o[m][t];
      }
      if (w == 0 && q4 == 0) {
        a.ml[pr * 2] = m_run[m];
        a.ml[pr * 2 + 1] = l;
      }
    }
  }
}

// one workgroup per row; up to MAX_SPLITS ranges
constexpr int MAX_SPLITS = 1024;
__global__ void __launch_bounds__(128) latent_combine_kernel(const float* __restrict__ acc, const float* __restrict__ ml,
                                                             const float* __restrict__ sink, bf16* __restrict__ out,
                                                             int64_t rows, int H, int R, int splits) {
  __shared__ float wt[MAX_SPLITS];
  __shared__ float red[2];
  const int64_t r = blockIdx.x;
  const float sk = sink ? sink[r % H] * LOG2E : -INFINITY;
  float M = sk, den = 0.f;
  for (int s = threadIdx.x; s < splits; s += 128) {
    wt[s] = ml[(s * rows + r) * 2];
    M = fmaxf(M, wt[s]);
  }
  M = block_max(M, red);
  for (int s = threadIdx.x; s < splits; s += 128) {
    wt[s] = exp2f(wt[s] - M);  // 0 for ranges that had nothing to add, and wrote nothing
    den = fmaf(wt[s], ml[(s * rows + r) * 2 + 1], den);
  }
  den = block_sum(den, red) + exp2f(sk - M);  // (its barriers publish the weights)
  for (int c = threadIdx.x * 4; c < R; c += 512) {
    const float* a = acc + r * R + c;
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
    for (int s = 0; s < splits; ++s) {
      const f32x4 x = *reinterpret_cast<const f32x4*>(a + s * rows * R);
      const float w = wt[s];
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = w > 0.f ? fmaf(x[j], w, v[j]) : v[j];
    }
    bf16x4 o;
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = (bf16)(v[j] / den);
    *reinterpret_cast<bf16x4*>(out + r * R + c) = o;
  }
}

size_t lds_bytes(int mr, int W) {
  const int KP = ((W + 31) & ~31) + 8, rows = 16 * mr;
  return (size_t)(BN + rows) * KP * 2 + 2 * rows * PP * 2 + 4 * rows * 4;
}

template <int MR, int NV>
int launch(const LatArgs& a, int nseq, int blocks, hipStream_t st) {
  static bool attr = false;
  if (!attr) {
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_decode_kernel<MR, NV>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    attr = true;
  }
  hipLaunchKernelGGL((latent_decode_kernel<MR, NV>), dim3(nseq, blocks, a.splits), dim3(NT), lds_bytes(MR, a.R + a.r), st, a);
  DS_CHECK_LAUNCH();
  return 0;
}

constexpr size_t LDS_MAX = 160 * 1024;
int row_tiles(int max_rows, int W) { return max_rows <= 16 ? 1 : max_rows <= 32 || lds_bytes(4, W) > LDS_MAX ? 2 : 4; }
// value tiles per wave and row pieces a kernel instance holds
int nv_of(int R) { return R <= 64 ? 1 : R <= 128 ? 2 : R <= 256 ? 4 : 8; }
int pieces_of(int nv) { return nv == 1 ? 16 : nv == 2 ? 24 : nv == 4 ? 40 : 72; }

}  // namespace

extern "C" int ds_latent_decode_ok(int R, int r) {
  return R > 0 && R % 8 == 0 && r >= 0 && r % 8 == 0 && R <= 512 && (R + r) / 8 <= pieces_of(nv_of(R));
}

// Keys per range and number of ranges for `nseq` sequences of up to max_new tokens and max_len keys in sight of them
extern "C" void ds_latent_decode_plan(int nseq, int max_new, int H, int W, int max_len, int* range, int* splits) {
  const int rows = max_new * H, per = 16 * row_tiles(rows, W), blocks = (rows + per - 1) / per;
  const int tiles = (max_len + BN - 1) / BN;
  // as many workgroups as the chip's LDS holds at once: a second, partly filled round would cost as much as the first
  const int resident = 256 * (int)(LDS_MAX / lds_bytes(row_tiles(rows, W), W));
  int want = (resident < 1024 ? resident : 1024) / (nseq * blocks);
  if (want > tiles) want = tiles;
  if (want < 1) want = 1;
  const int per_range = (tiles + want - 1) / want;
  *range = per_range * BN;
  *splits = (tiles + per_range - 1) / per_range;
}

// Sequences first .. first + nseq of the tables, none with more than max_new tokens; their `tokens` tokens begin with the
// batch's token tok_base. q [tokens, H, R + r], lat [blocks, BS, R + r] -> out [tokens, H, R]. acc / ml: workspace of `splits` ranges (unused with one).
extern "C" int ds_latent_decode(const void* q, const void* lat, void* out, float* acc, float* ml, const int* bt, int max_blocks,
                                const int* cu, const int* start, int first, int nseq, int max_new, int tok_base, int tokens, int H, int R,
                                int r, int BS, int range, int splits, int window, const float* sink, float scale, hipStream_t st) {
  if (nseq <= 0) return 0;
  if (!ds_latent_decode_ok(R, r) || H <= 0 || BS <= 0 || max_blocks <= 0 || range <= 0 || range % BN || splits <= 0 ||
      splits > MAX_SPLITS || max_new <= 0 || tokens <= 0 || window < 0 || (splits > 1 && (!acc || !ml)))
    return (int)hipErrorInvalidValue;
  const LatArgs a{(const bf16*)q, (const bf16*)lat, (bf16*)out, acc, ml, bt, cu, start, sink, first, tok_base, H, R, r, BS,
                  max_blocks, range, splits, window, (int64_t)tokens * H, scale * LOG2E};
  const int mr = row_tiles(max_new * H, R + r);
  const int blocks = (max_new * H + 16 * mr - 1) / (16 * mr);
  if (blocks > 65535) return (int)hipErrorInvalidValue;
  int rc = (int)hipErrorInvalidValue;
#define ROW(NV)                                        \
  {                                                    \
    if (mr == 1) rc = launch<1, NV>(a, nseq, blocks, st); \
    else if (mr == 2) rc = launch<2, NV>(a, nseq, blocks, st); \
    else rc = launch<4, NV>(a, nseq, blocks, st);      \
  }
  switch (nv_of(R)) {
    case 1: ROW(1) break;
    case 2: ROW(2) break;
    case 4: ROW(4) break;
    default: ROW(8)
  }
#undef ROW
  if (rc) return rc;
  if (splits > 1) {
    hipLaunchKernelGGL(latent_combine_kernel, dim3((unsigned)a.rows), dim3(128), 0, st, acc, ml, sink, (bf16*)out, a.rows, H,
                       R, splits);
    DS_CHECK_LAUNCH();
  }
  return 0;
}
