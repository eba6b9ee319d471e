// Recurrences with a scalar decay per head over long portions, by chunks of 64 (or 32) tokens (CDNA4, gfx950). See decayed_scan.hip
// for the recurrence.
//
// With the running log decay G_i of a chunk (its first token included) and the state S0 the chunk starts from:
//     o_i = e^{G_i} S0^T q_i + sum_{j <= i} P_ij v_j + D v_i,    P_ij = e^{G_i - G_j} b_j (q_i . k_j)
//     S   = e^{G_C} S0 + sum_j e^{G_C - G_j} b_j k_j v_j^T
// (the first two terms of o times a constant). The normaliser's products are the same with a single value column of ones:
// z . q_i = e^{G_i} z0 . q_i + sum_j P_ij. Every workgroup keeps its own, moved on by one of its pairs of waves.
// One workgroup per (sequence, head, 16 WC value columns) walks the chunks. Two of its 2 WC waves share 16 value columns: each
// keeps half of the key rows of their state in registers, in the result layout of the matrix instructions. The next state
// accumulates into it, and the same registers are the left operand of the read-out (a product's k order is free as long as
// both sides agree on it). The two halves of the read-out meet in LDS, where the 64 x 64 weights P are shared too.
//
// Precision: q, k and v are bf16 activations, or q and k (where they were computed on, as by a rotation) sums of two bf16 terms;
// everything else is fp32. The bf16 matrix instructions take an fp32 operand
// as three bf16 terms (8 + 8 + 8 mantissa bits, nothing is lost) with fp32 accumulation, so state, weights and decays
// enter the products as 32-bit numbers at a third of the bf16 rate, five times that of the fp32 instructions. Log decays
// are summed in fp64: only differences enter, and a strong decay early in a chunk must not cost the later ones their digits.
// The chunk borders are counted from the portion's first token; where they fall changes rounding only.
#include "decayed_scan.h"

namespace {

// Tokens per chunk. 32 where two terms of q and k fill the LDS, or a wide normaliser the registers
constexpr int chunk_of(int NK, bool NORM, int QT) { return (QT == 2 && NK >= 4) || (NORM && NK > 4) ? 32 : 64; }
constexpr double LOG2E = 1.4426950408889634073599246810019;

typedef short s16x4_t __attribute__((ext_vector_type(4)));
typedef unsigned u32x4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ f32x4 mfma(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
// Workgroup barrier for LDS: earlier LDS accesses have completed, global loads may still be under way
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// Upper halves of two words side by side: two fp32 numbers cut to bf16
__device__ __forceinline__ unsigned pack_hi(unsigned lo, unsigned hi) { return __builtin_amdgcn_perm(hi, lo, 0x07060302u); }

// Pairs of fp32 numbers as the sums of three bf16 numbers each: the leading 8 mantissa bits, the next 8, the rest (exact)
__device__ __forceinline__ void split3(float x, float y, unsigned& a, unsigned& b, unsigned& c) {
  const unsigned xi = __float_as_uint(x), yi = __float_as_uint(y);
  const float xr = x - __uint_as_float(xi & 0xffff0000u), yr = y - __uint_as_float(yi & 0xffff0000u);
  const unsigned xj = __float_as_uint(xr), yj = __float_as_uint(yr);
  a = pack_hi(xi, yi);
  b = pack_hi(xj, yj);
  c = pack_hi(__float_as_uint(xr - __uint_as_float(xj & 0xffff0000u)), __float_as_uint(yr - __uint_as_float(yj & 0xffff0000u)));
}
// The same for the 8 elements of an operand
__device__ __forceinline__ void split3(const float (&x)[8], bf16x8& a, bf16x8& b, bf16x8& c) {
  u32x4_t u, v, w;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    unsigned p, q, r;
    split3(x[2 * i], x[2 * i + 1], p, q, r);
    u[i] = p;
    v[i] = q;
    w[i] = r;
  }
  a = __builtin_bit_cast(bf16x8, u);
  b = __builtin_bit_cast(bf16x8, v);
  c = __builtin_bit_cast(bf16x8, w);
}

// Sum over the lanes that share lane % 16, in all of them
__device__ __forceinline__ float sum_rows16(float x) {
  auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(x), false, false);  // rows (0 0 2 2), (1 1 3 3)
  x = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  a = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  return __uint_as_float(a[0]) + __uint_as_float(a[1]);
}

// by value: a choice between array elements must not become one between addresses
__device__ __forceinline__ f32x4 pick(bool c, f32x4 a, f32x4 b) {
  f32x4 r;
#pragma unroll
  for (int i = 0; i < 4; ++i) r[i] = c ? a[i] : b[i];
  return r;
}

// Operand whose lane wants one column of 8 rows: rows r .. r + 3 and r2 .. r2 + 3 of 16 columns from `col` on, transposed
// on the way out of LDS. `i` is the lane within its group of 16.
__device__ __forceinline__ bf16x8 read_tr(const bf16* base, int pitch, int r, int r2, int col, int i) {
  auto at = [&](int row) {
    return __builtin_amdgcn_ds_read_tr16_b64_v4i16(
        (__attribute__((address_space(3))) s16x4_t*)(base + (row + (i >> 2)) * pitch + col + 4 * (i & 3)));
  };
  const s16x4_t lo = at(r), hi = at(r2);
  s16x8 v;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    v[e] = lo[e];
    v[4 + e] = hi[e];
  }
  return __builtin_bit_cast(bf16x8, v);
}

// NK: 32-wide steps of the key width (rounded up), even unless the waves of a pair cannot share (NK 1: the second one has
// no rows); WC: groups of 16 value columns; NORM: with a normaliser; QT: terms of q and k
template <int NK, int WC, bool NORM, int QT>
__global__ void __launch_bounds__(128 * WC, (NK <= 4 || WC == 4 ? 2 : 1)) decayed_chunk_kernel(
    const bf16* __restrict__ qk, const bf16* __restrict__ v, const float* __restrict__ gb,
    const float* __restrict__ log_decay, const float* __restrict__ skip, float scale, const bf16* __restrict__ proj,
    float* __restrict__ state, float* __restrict__ zstate, const float* __restrict__ floors, bf16* __restrict__ conv_state,
    const int* __restrict__ seqs, const int* __restrict__ cu, const int* __restrict__ start, const int* __restrict__ slots, bf16* __restrict__ out, ScanDims D) {
  constexpr int C = chunk_of(NK, NORM, QT), PP = C + 8;   // PP: LDS row length of the weights
  constexpr int NT = 128 * WC, NW = 2 * WC, VT = 16 * WC, FT = C / 32;  // FT: token tiles a wave finishes
  constexpr int KP = 32 * NK + 8, VP = VT + 8;      // LDS row lengths of q and k, of v
  constexpr int KH = (NK + 1) / 2;                  // steps of a wave's half of the key rows
  constexpr int PQ = C * 4 * NK / NT, PV = (C * VT / 8 + NT - 1) / NT;  // 16-byte pieces per thread of q or k, of v
  static_assert(C * 4 * NK % NT == 0 || NK == 1, "pieces");
  constexpr int PQN = PQ > 0 ? PQ : 1;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  bf16* const Qs = reinterpret_cast<bf16*>(smem);                 // [QT][C][KP]
  bf16* const Ks = Qs + QT * C * KP;
  bf16* const Vs = Ks + QT * C * KP;
  bf16* const Ps = Vs + C * VP;                                   // [3][C][PP]
  f32x4* const Ys = reinterpret_cast<f32x4*>(Ps + 3 * C * PP);    // [NW][FT][64]: halves of the read-out on their way
  double* const Gs = reinterpret_cast<double*>(Ys + NW * FT * 64); // [2 NW][C] running log2 decay
  float* const bs = reinterpret_cast<float*>(Gs + 2 * NW * C);    // [2 NW][C] step sizes
  float* const eg = bs + 2 * NW * C;                              // [2 NW][C] e^{G_i}
  float* const ws = eg + 2 * NW * C;                              // [2 NW][C] e^{G_C - G_j} b_j
  float* const fl = ws + 2 * NW * C;                              // NORM: [2 NW][C] floors,
  float* const zs = fl + 2 * NW * C;                              //   [2][32 NK] normaliser the chunk starts from,
  float* const zq = zs + 64 * NK;                                 //   [C] its products with the queries,
  float* const rs = zq + C;                                       //   [4][C] sums of P's rows over 16 columns each

  const int vts = (D.dv + VT - 1) / VT, bid = xcd_remap(blockIdx.x, gridDim.x);
  const int vt = bid % vts, h = bid / vts % D.H, seq = seqs[2 * (bid / (vts * D.H))];
  const int g = h / (D.H / D.Hk), tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, q4 = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6), wc = w >> 1, half = w & 1;
  const int t0 = cu[seq], n = cu[seq + 1] - t0, nc = (n + C - 1) / C, v0 = vt * VT, dks = D.dks(), dvs = D.dvs();
  const bool fresh = start[seq] == 0;
  const int col = v0 + 16 * wc + l16;  // this lane's column of the state
  const int k_first = half * KH * 32;  // first key row of the wave's half (NK 1: rows 32 .. 63 do not exist)
  const bool rows_ok = half * KH < NK;
  float* st = state + (((int64_t)slots[seq] * D.H + h) * D.dv + min(col, D.dv - 1)) * dks;

  f32x4 S[2 * KH];  // rows k_first + 16 t + 4 q4 + 0..3
  f32x4 Z[NORM ? 2 * KH : 1];
#pragma unroll
  for (int t = 0; t < 2 * KH; ++t) {
    const int k = k_first + 16 * t + 4 * q4;
    S[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (!fresh && col < D.dv && k < dks) S[t] = *reinterpret_cast<const f32x4*>(st + k);
  }
  if constexpr (NORM) {  // (visible after the first barrier of the loop)
    const float* zt = zstate + D.z_at(slots[seq], h, v0);
    for (int k = tid; k < 32 * NK; k += NT) zs[k] = !fresh && k < dks ? zt[k] : 0.f;
#pragma unroll
    for (int t = 0; t < 2 * KH; ++t) {
      const int k = k_first + 16 * t + 4 * q4;
      Z[t] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (!fresh && k < dks) Z[t] = *reinterpret_cast<const f32x4*>(zt + k);
    }
  }
  const float sk = skip ? skip[h] : 0.f, ld = log_decay ? log_decay[h] : 0.f;
  const bf16* qbase = qk + D.q_at(g, t0);
  const bf16* kbase = qk + D.k_at(g, t0);
  const bf16* vbase = v + D.v_at(h, t0) + v0;
  const int64_t term = 2 * D.Hk * D.T * dks;  // from one term of q and k to the next
  const int vw = min(dvs - v0, VT);    // v columns of this workgroup that exist
  const bool k_full = dks == 32 * NK, v_full = vw == VT;

  // ---- a chunk's rows on their way to LDS: 4 NK (q, k) and VT / 8 (v) 16-byte pieces per row
  bf16x8 rq[QT][PQN], rk[QT][PQN], rv[PV];
  auto fetch = [&](int c) {
    const bool whole = (c + 1) * C <= n;
    const int64_t base = (int64_t)c * C * dks, vb = (int64_t)c * C * dvs;
    const int last = n - 1 - c * C;
#pragma unroll
    for (int i = 0; i < PQN; ++i) {
      const int p = tid + i * NT;
      int row = p / (4 * NK), ch = p % (4 * NK) * 8;
      if (!whole) row = min(row, last);
      if (!k_full) ch = min(ch, dks - 8);
      if (PQ > 0 || p < C * 4 * NK) {
#pragma unroll
        for (int u = 0; u < QT; ++u) {
          rq[u][i] = *reinterpret_cast<const bf16x8*>(qbase + u * term + base + row * dks + ch);
          rk[u][i] = *reinterpret_cast<const bf16x8*>(kbase + u * term + base + row * dks + ch);
        }
      }
    }
#pragma unroll
    for (int i = 0; i < PV; ++i) {
      const int p = tid + i * NT;
      int row = p / (VT / 8), ch = p % (VT / 8) * 8;
      if (!whole) row = min(row, last);
      if (!v_full) ch = min(ch, vw - 8);
      if (p < C * VT / 8) rv[i] = *reinterpret_cast<const bf16x8*>(vbase + vb + row * dvs + ch);
    }
  };
  auto stage = [&](int c) {  // rows past the portion's end and columns past the widths become zero
    const bool whole = (c + 1) * C <= n;
    bf16x8 z;
#pragma unroll
    for (int e = 0; e < 8; ++e) z[e] = (bf16)0.f;
    if (!whole || !k_full || !v_full) {
#pragma unroll
      for (int i = 0; i < PQN; ++i) {
        const int p = tid + i * NT;
        if (c * C + p / (4 * NK) >= n || p % (4 * NK) * 8 >= dks) {
#pragma unroll
          for (int u = 0; u < QT; ++u) rq[u][i] = rk[u][i] = z;
        }
      }
#pragma unroll
      for (int i = 0; i < PV; ++i) {
        const int p = tid + i * NT;
        if (c * C + p / (VT / 8) >= n || p % (VT / 8) * 8 >= vw) rv[i] = z;
      }
    }
#pragma unroll
    for (int i = 0; i < PQN; ++i) {
      const int p = tid + i * NT, row = p / (4 * NK), ch = p % (4 * NK) * 8;
      if (PQ > 0 || p < C * 4 * NK) {
#pragma unroll
        for (int u = 0; u < QT; ++u) {
          *reinterpret_cast<bf16x8*>(Qs + (u * C + row) * KP + ch) = rq[u][i];
          *reinterpret_cast<bf16x8*>(Ks + (u * C + row) * KP + ch) = rk[u][i];
        }
      }
    }
#pragma unroll
    for (int i = 0; i < PV; ++i) {
      const int p = tid + i * NT;
      if (p < C * VT / 8) *reinterpret_cast<bf16x8*>(Vs + p / (VT / 8) * VP + p % (VT / 8) * 8) = rv[i];
    }
  };
  // ---- decays and step sizes of a chunk, a lane per token (the others add nothing): every NW chunks each wave prepares one of the next NW
  float lg = 0.f, lb = 0.f, lf = 0.f;
  auto fetch_gb = [&](int c) {
    const int64_t t = t0 + min(c * C + lane, n - 1);
    lg = gb ? gb[t * 2 * D.H + h] : ld;
    lb = gb ? gb[(t * 2 + 1) * D.H + h] : 1.f;
    if constexpr (NORM) lf = floors[t * D.H + h];
  };
  auto scan_gb = [&](int c) {
    const bool ok = lane < C && c * C + lane < n;  // rows past the end neither decay nor add anything
    const float b0 = ok ? lb : 0.f;
    double G = ok ? (double)lg * LOG2E : 0.0;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const double p = __shfl_up(G, o, 64);
      if (lane >= o) G += p;
    }
    const double GC = __shfl(G, 63, 64);
    if (lane >= C) return;
    const int b = c % (2 * NW) * C + lane;
    Gs[b] = G;
    bs[b] = b0;
    eg[b] = __builtin_amdgcn_exp2f((float)G);
    ws[b] = __builtin_amdgcn_exp2f((float)(GC - G)) * b0;
    if constexpr (NORM) fl[b] = lf;
  };
  fetch(0);
  fetch_gb(w);
  scan_gb(w);
  for (int c = 0; c < nc; ++c) {
    const int cb = c % (2 * NW) * C;
    const bool ahead = c % NW == 0 && c + NW < nc;
    stage(c);
    if (c + 1 < nc) fetch(c + 1);
    if (ahead) fetch_gb(c + NW + w);
    lds_barrier();
    // ---- P. The read-out takes pairs of 16 x 16 tiles of a row: 10 tiles up to the diagonal, and 2 behind it that are zero
    // (32 tokens: 3 and 1)
    constexpr int PT = C == 64 ? 12 : 4;
#pragma unroll
    for (int u = 0; u < (PT + NW - 1) / NW; ++u) {
      const int tl = w + u * NW;
      if (tl >= PT) break;
      const int it = tl < 4 ? tl >> 1 : 2 + ((tl - 4) >> 2), jt = tl < 4 ? tl & 1 : (tl - 4) & 3;
      f32x4 s = {0.f, 0.f, 0.f, 0.f};
      if (jt <= it) {
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) {
          const bf16 *kr = Ks + (16 * jt + l16) * KP + 32 * kk + 8 * q4, *qr = Qs + (16 * it + l16) * KP + 32 * kk + 8 * q4;
          const bf16x8 k0 = *reinterpret_cast<const bf16x8*>(kr), q0 = *reinterpret_cast<const bf16x8*>(qr);
          if constexpr (QT == 2) {  // (the product of the second terms is below 2^-16 of the whole)
            s = mfma(*reinterpret_cast<const bf16x8*>(kr + C * KP), q0, s);
            s = mfma(k0, *reinterpret_cast<const bf16x8*>(qr + C * KP), s);
          }
          s = mfma(k0, q0, s);
        }
        // lane: row i of P, columns j .. j + 3
        const int i = 16 * it + l16, j = 16 * jt + 4 * q4;
        const double gi = Gs[cb + i];
#pragma unroll
        for (int r = 0; r < 4; ++r)
        {  // (no branch: behind the diagonal the factor is some number, or infinite)
          const float f = s[r] * (__builtin_amdgcn_exp2f((float)(gi - Gs[cb + j + r])) * bs[cb + j + r]);
          s[r] = j + r <= i ? f : 0.f;
        }
        if constexpr (NORM) {
          const float sum = sum_rows16((s[0] + s[1]) + (s[2] + s[3]));
          if (q4 == 0) rs[jt * C + i] = sum;
        }
      }
      unsigned a[2], b[2], d[2];
      split3(s[0], s[1], a[0], b[0], d[0]);
      split3(s[2], s[3], a[1], b[1], d[1]);
      bf16* p = Ps + (16 * it + l16) * PP + 16 * jt + 4 * q4;
      *reinterpret_cast<uint2*>(p) = uint2{a[0], a[1]};
      *reinterpret_cast<uint2*>(p + C * PP) = uint2{b[0], b[1]};
      *reinterpret_cast<uint2*>(p + 2 * C * PP) = uint2{d[0], d[1]};
    }
    // ---- read-out of the state the chunk starts from, this half of the key rows: y^T [16 columns, 64 tokens] = S^T q^T
    f32x4 y[2 * FT];
#pragma unroll
    for (int i = 0; i < 2 * FT; ++i) y[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (rows_ok) {
#pragma unroll
      for (int kk = 0; kk < KH; ++kk) {
        bf16x8 s0, s1, s2;  // k slot 8 q4 + e is key row k_first + 32 kk + 16 (e / 4) + 4 q4 + e % 4
        float x[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = S[2 * kk + (e >> 2)][e & 3];
        split3(x, s0, s1, s2);
#pragma unroll
        for (int i = 0; i < 2 * FT; ++i) {
          const bf16* qr = Qs + (16 * i + l16) * KP + k_first + 32 * kk + 4 * q4;
          auto row = [&](const bf16* p) {
            const bf16x4 lo = *reinterpret_cast<const bf16x4*>(p), hi = *reinterpret_cast<const bf16x4*>(p + 16);
            bf16x8 q;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              q[e] = lo[e];
              q[4 + e] = hi[e];
            }
            return q;
          };
          if constexpr (QT == 2) {
            const bf16x8 qc = row(qr + C * KP);
            y[i] = mfma(s1, qc, y[i]);
            y[i] = mfma(s0, qc, y[i]);
          }
          const bf16x8 qb = row(qr);
          y[i] = mfma(s2, qb, y[i]);
          y[i] = mfma(s1, qb, y[i]);
          y[i] = mfma(s0, qb, y[i]);
        }
      }
    }
    float* const zc = zs + (c & 1) * 32 * NK;        // NORM: this chunk's normaliser, the next one's
    float* const zn = zs + ((c & 1) ^ 1) * 32 * NK;
    if constexpr (NORM) {  // z0 . q: neighbouring lanes share a token, 8 key columns at a time
      constexpr int LP = NT / C;
      const int row = tid / LP, part = tid % LP;
      float a = 0.f;
      for (int k = 8 * part; k < 32 * NK; k += 8 * LP) {
        float x[8], y[8];
        Vec8<bf16>::load(Qs + row * KP + k, x);
        Vec8<float>::load(zc + k, y);
#pragma unroll
        for (int e = 0; e < 8; ++e) a = fmaf(x[e], y[e], a);
      }
#pragma unroll
      for (int o = 1; o < LP; o <<= 1) a += __shfl_xor(a, o, 64);
      if (part == 0) zq[row] = a;
    }
    // each wave of a pair finishes half of the token tiles: the others go to its partner
#pragma unroll
    for (int i = 0; i < FT; ++i) Ys[(w * FT + i) * 64 + lane] = pick(half, y[i], y[FT + i]);
    // this pair's columns of v: lane l16 a column, tokens 32 s + 8 q4 + e
    bf16x8 vf[FT];
#pragma unroll
    for (int s = 0; s < FT; ++s) vf[s] = read_tr(Vs, VP, 32 * s + 8 * q4, 32 * s + 8 * q4 + 4, 16 * wc, l16);
    // ---- next state
    if (rows_ok) {
      const float dc = eg[cb + C - 1];
#pragma unroll
      for (int s = 0; s < FT; ++s) {
        bf16x8 u0, u1, u2;
        float x[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = (float)vf[s][e] * ws[cb + 32 * s + 8 * q4 + e];
        split3(x, u0, u1, u2);
        bf16x8 z0, z1, z2;  // the first pair's waves move the normaliser on too, 16 times the same column
        if (NORM && wc == 0) {
#pragma unroll
          for (int e = 0; e < 8; ++e) x[e] = ws[cb + 32 * s + 8 * q4 + e];
          split3(x, z0, z1, z2);
        }
#pragma unroll
        for (int t = 0; t < 2 * KH; ++t) {
          const bf16x8 kf = read_tr(Ks, KP, 32 * s + 8 * q4, 32 * s + 8 * q4 + 4, k_first + 16 * t, l16);
          if (s == 0) S[t] *= dc;
          if constexpr (QT == 2) {
            const bf16x8 kl = read_tr(Ks + C * KP, KP, 32 * s + 8 * q4, 32 * s + 8 * q4 + 4, k_first + 16 * t, l16);
            S[t] = mfma(kl, u1, S[t]);
            S[t] = mfma(kl, u0, S[t]);
          }
          S[t] = mfma(kf, u2, S[t]);
          S[t] = mfma(kf, u1, S[t]);
          S[t] = mfma(kf, u0, S[t]);
          if (NORM && wc == 0) {
            if (s == 0) Z[t] *= dc;
            Z[t] = mfma(kf, z2, Z[t]);
            Z[t] = mfma(kf, z1, Z[t]);
            Z[t] = mfma(kf, z0, Z[t]);
          }
        }
      }
    }
    if (NORM && wc == 0 && rows_ok && l16 == 0) {
#pragma unroll
      for (int t = 0; t < 2 * KH; ++t) *reinterpret_cast<f32x4*>(zn + k_first + 16 * t + 4 * q4) = Z[t];
    }
    lds_barrier();  // P and the partner's half are complete
    // ---- within the chunk, this wave's token tiles
#pragma unroll
    for (int k = 0; k < FT; ++k) {
      const int i = FT * half + k;
      f32x4 acc = pick(half, y[FT + k], y[k]);
      acc = (acc + Ys[((w ^ 1) * FT + k) * 64 + lane]) * eg[cb + 16 * i + l16];
#pragma unroll
      for (int s = 0; s < FT; ++s) {
        if (s > i / 2) break;
        const bf16* pr = Ps + (16 * i + l16) * PP + 32 * s + 8 * q4;
        acc = mfma(vf[s], *reinterpret_cast<const bf16x8*>(pr + 2 * C * PP), acc);
        acc = mfma(vf[s], *reinterpret_cast<const bf16x8*>(pr + C * PP), acc);
        acc = mfma(vf[s], *reinterpret_cast<const bf16x8*>(pr), acc);
      }
      if constexpr (NORM) {
        const int r = 16 * i + l16;
        float z = eg[cb + r] * zq[r];
#pragma unroll
        for (int jt = 0; jt < C / 16; ++jt) {  // (tiles behind the diagonal hold leftovers)
          const float p = rs[jt * C + r];
          z += jt <= i ? p : 0.f;
        }
        acc *= scale / (fmaxf(fabsf(z * scale), fl[cb + r]) + 1e-6f);
      } else {
        acc *= scale;
      }
      const int t = c * C + 16 * i + l16, cv = v0 + 16 * wc + 4 * q4;
      const bf16x4 vv = *reinterpret_cast<const bf16x4*>(Vs + (16 * i + l16) * VP + 16 * wc + 4 * q4);
      bf16x4 o;
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = (bf16)fmaf(sk, (float)vv[r], acc[r]);
      bf16* dst = out + ((int64_t)(t0 + t) * D.H + h) * D.dv + cv;
      if (D.dv % 4 == 0) {
        if (t < n && cv < D.dv) *reinterpret_cast<bf16x4*>(dst) = o;
      } else if (t < n) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (cv + r < D.dv) dst[r] = o[r];
      }
    }
    if (ahead) scan_gb(c + NW + w);
    lds_barrier();
  }
  if (col < D.dv) {
#pragma unroll
    for (int t = 0; t < 2 * KH; ++t) {
      const int k = k_first + 16 * t + 4 * q4;
      if (k < dks) *reinterpret_cast<f32x4*>(st + k) = S[t];
    }
  }
  if constexpr (NORM) {  // (the loop ends with a barrier) every copy that is about this workgroup's columns
    for (int cc = 0; cc < VT && v0 + cc < D.dv; cc += Z_COLS) {
      float* zt = zstate + D.z_at(slots[seq], h, v0 + cc);
      for (int k = tid; k < dks; k += NT) zt[k] = zs[(nc & 1) * 32 * NK + k];
    }
  }
  if (vt == 0 && D.taps > 1)
    advance_windows(conv_state + (int64_t)slots[seq] * (D.taps - 1) * D.channels, proj, t0, n, D, fresh, h);
}

template <int NK, int WC, bool NORM, int QT>
int launch(const void* qk, const void* v, const float* gb, const float* log_decay, const float* skip, float scale,
           const void* proj, float* state, float* zstate, const float* floors, void* conv_state, const int* seqs, int nseq, const int* cu, const int* start, const int* slots,
           void* out, const ScanDims& D, hipStream_t st) {
  constexpr int VT = 16 * WC, C = chunk_of(NK, NORM, QT);
  constexpr int LDS = (2 * QT * C * (32 * NK + 8) + C * (VT + 8) + 3 * C * (C + 8)) * 2 + 2 * WC * C / 32 * 64 * 16 +
                      4 * WC * C * 20 +
                      (NORM ? (4 * WC * C + 64 * NK + 5 * C) * 4 : 0);
  static bool attr = false;
  if (!attr) {
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&decayed_chunk_kernel<NK, WC, NORM, QT>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, LDS);
    attr = true;
  }
  hipLaunchKernelGGL((decayed_chunk_kernel<NK, WC, NORM, QT>), dim3((unsigned)((D.dv + VT - 1) / VT * D.H * nseq)), dim3(128 * WC), LDS,
                     st, (const bf16*)qk, (const bf16*)v, gb, log_decay, skip, scale, (const bf16*)proj, state, zstate,
                     floors, (bf16*)conv_state, seqs, cu, start, slots, (bf16*)out, D);
  DS_CHECK_LAUNCH();
  return 0;
}

}  // namespace

extern "C" int ds_scan_chunk_ok(int dk) { return dk <= 256; }

// bf16 storage, dk up to 256. seqs [nseq, 2]: (sequence, anything). zstate, floors, terms: as for ds_scan_recur
extern "C" int ds_scan_chunk(const void* qk, const void* v, const float* gb, const float* log_decay, const float* skip,
                             float scale, const void* proj, float* state, float* zstate, const float* floors,
                             void* conv_state, int terms, const int* seqs, int nseq, const int* cu,
                             const int* start, const int* slots, void* out, const int* dims, int tokens, hipStream_t st) {
  if (nseq <= 0) return 0;
  const ScanDims D{dims[0], dims[1], dims[2], dims[3], dims[4], dims[5], dims[6], dims[7], dims[8], dims[9], dims[10], dims[11],
                   tokens};
  if (!scan_dims_ok(D) || !ds_scan_chunk_ok(D.dk) || (!gb == !log_decay) || (!zstate != !floors) ||
      terms < 1 || terms > 2 || (terms == 2 && zstate) || (D.taps > 1 && !conv_state) ||
      (int64_t)nseq * D.H * ((D.dv + 31) / 32) > INT32_MAX)
    return (int)hipErrorInvalidValue;
  // wide workgroups share q, k and P among more columns; narrow ones where there are too few to fill the chip
  const bool wide = D.dv > 32 && (int64_t)nseq * D.H * ((D.dv + 63) / 64) >= 192;
#define RUN(NK, WC, NORM, QT)                                                                                           \
  return launch<NK, WC, NORM, QT>(qk, v, gb, log_decay, skip, scale, proj, state, zstate, floors, conv_state, seqs, nseq, cu, \
                                  start, slots, out, D, st)
#define GO(NK)                                    \
  {                                               \
    if (terms == 2 && wide) RUN(NK, 4, false, 2); \
    if (terms == 2) RUN(NK, 2, false, 2);         \
    if (zstate && wide) RUN(NK, 4, true, 1);      \
    if (zstate) RUN(NK, 2, true, 1);              \
    if (wide) RUN(NK, 4, false, 1);               \
    RUN(NK, 2, false, 1);                         \
  }
  if (D.dk <= 32) GO(1)
  if (D.dk <= 64) GO(2)
  if (D.dk <= 128) GO(4)
  GO(8)
#undef GO
#undef RUN
}
