// Recurrences with a scalar decay per head over long portions, by chunks of 64 tokens (CDNA4, gfx950). See decayed_scan.hip
// for the recurrence.
//
// With the running log decay G_i of a chunk (its first token included) and the state S0 the chunk starts from:
//     o_i = e^{G_i} S0^T q_i + sum_{j <= i} P_ij v_j + D v_i,    P_ij = e^{G_i - G_j} b_j (q_i . k_j)
//     S   = e^{G_C} S0 + sum_j e^{G_C - G_j} b_j k_j v_j^T
// One workgroup per (sequence, head, 64 value columns) walks the chunks. Each of its four waves owns 16 value columns and
// keeps their state [dk, 16] in registers, in the result layout of the matrix instructions: the next state accumulates
// into it, and the same registers are the left operand of the read-out (a product's k order is free as long as both sides
// agree on it). The 64 x 64 weights P are computed once per workgroup and shared through LDS.
//
// Precision: q, k and v are bf16 activations; everything else is fp32. The bf16 matrix instructions take an fp32 operand
// as three bf16 terms (8 + 8 + 8 mantissa bits, nothing is lost) with fp32 accumulation, so state, weights and decays
// enter the products as 32-bit numbers at a third of the bf16 rate, five times that of the fp32 instructions. Log decays
// are summed in fp64: only differences enter, and a strong decay early in a chunk must not cost the later ones their digits.
// The chunk borders are counted from the portion's first token; where they fall changes rounding only.
#include "decayed_scan.h"

namespace {

constexpr int C = 64;
constexpr int NT = 256;
constexpr int VT = 64;       // value columns per workgroup
constexpr int VP = VT + 8;   // LDS row lengths (elements)
constexpr int PP = C + 8;

typedef short s16x4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ f32x4 mfma(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
// Workgroup barrier for LDS: earlier LDS accesses have completed, global loads may still be under way
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// x as three bf16 terms
__device__ __forceinline__ void split3(float x, bf16& a, bf16& b, bf16& c) {
  a = (bf16)x;
  const float r = x - (float)a;
  b = (bf16)r;
  c = (bf16)(r - (float)b);
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

// NK: 32-wide steps of the key width (rounded up)
template <int NK>
__global__ void __launch_bounds__(NT, (NK <= 4 ? 2 : 1)) decayed_chunk_kernel(
    const bf16* __restrict__ qk, const bf16* __restrict__ v, const float* __restrict__ gb,
    const float* __restrict__ log_decay, const float* __restrict__ skip, const bf16* __restrict__ proj,
    float* __restrict__ state, bf16* __restrict__ conv_state, const int* __restrict__ seqs, const int* __restrict__ cu,
    const int* __restrict__ start, const int* __restrict__ slots, bf16* __restrict__ out, ScanDims D) {
  constexpr int KP = 32 * NK + 8;  // LDS row length of q and k
  extern __shared__ __attribute__((aligned(16))) char smem[];
  bf16* const Qs = reinterpret_cast<bf16*>(smem);
  bf16* const Ks = Qs + C * KP;
  bf16* const Vs = Ks + C * KP;
  bf16* const Ps = Vs + C * VP;                                   // [3][C][PP]
  double* const Gs = reinterpret_cast<double*>(Ps + 3 * C * PP);  // [2][C]
  float* const bs = reinterpret_cast<float*>(Gs + 2 * C);         // [2][C] step sizes
  float* const eg = bs + 2 * C;                                   // [2][C] e^{G_i}
  float* const ws = eg + 2 * C;                                   // [2][C] e^{G_C - G_j} b_j

  const int vts = (D.dv + VT - 1) / VT, bid = xcd_remap(blockIdx.x, gridDim.x);
  const int vt = bid % vts, h = bid / vts % D.H, seq = seqs[2 * (bid / (vts * D.H))];
  const int g = h / (D.H / D.Hk), tid = threadIdx.x, lane = tid & 63, w = tid >> 6, l16 = lane & 15, q4 = lane >> 4;
  const int t0 = cu[seq], n = cu[seq + 1] - t0, nc = (n + C - 1) / C, v0 = vt * VT, dks = D.dks(), dvs = D.dvs();
  const bool fresh = start[seq] == 0;
  const int col = v0 + 16 * w + l16;  // this lane's column of the state
  float* st = state + (((int64_t)slots[seq] * D.H + h) * D.dv + min(col, D.dv - 1)) * dks;

  f32x4 S[2 * NK];  // rows 16 t + 4 q4 + 0..3
#pragma unroll
  for (int t = 0; t < 2 * NK; ++t) {
    const int k = 16 * t + 4 * q4;
    S[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (!fresh && col < D.dv && k < dks) S[t] = *reinterpret_cast<const f32x4*>(st + k);
  }
  const float sk = skip ? skip[h] : 0.f, ld = log_decay ? log_decay[h] : 0.f;
  const bf16* qbase = qk + D.q_at(g, t0);
  const bf16* kbase = qk + D.k_at(g, t0);
  const bf16* vbase = v + D.v_at(h, t0);

  // ---- a chunk's rows on their way to LDS: 4 NK (q, k) and 8 (v) 16-byte pieces per row
  bf16x8 rq[NK], rk[NK], rv[2];
  auto fetch = [&](int c) {
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int p = tid + i * NT, row = p / (4 * NK), ch = p % (4 * NK) * 8;
      const int64_t off = (int64_t)min(c * C + row, n - 1) * dks + min(ch, dks - 8);
      rq[i] = *reinterpret_cast<const bf16x8*>(qbase + off);
      rk[i] = *reinterpret_cast<const bf16x8*>(kbase + off);
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int p = tid + i * NT, row = p / 8, ch = v0 + p % 8 * 8;
      rv[i] = *reinterpret_cast<const bf16x8*>(vbase + (int64_t)min(c * C + row, n - 1) * dvs + min(ch, dvs - 8));
    }
  };
  auto stage = [&](int c) {  // rows past the portion's end and columns past the widths become zero
    bf16x8 z;
#pragma unroll
    for (int e = 0; e < 8; ++e) z[e] = (bf16)0.f;
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int p = tid + i * NT, row = p / (4 * NK), ch = p % (4 * NK) * 8;
      const bool ok = c * C + row < n && ch < dks;
      *reinterpret_cast<bf16x8*>(Qs + row * KP + ch) = ok ? rq[i] : z;
      *reinterpret_cast<bf16x8*>(Ks + row * KP + ch) = ok ? rk[i] : z;
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int p = tid + i * NT, row = p / 8, ch = p % 8 * 8;
      *reinterpret_cast<bf16x8*>(Vs + row * VP + ch) = c * C + row < n && v0 + ch < dvs ? rv[i] : z;
    }
  };
  // ---- a chunk's decays and step sizes, a lane per token (one wave does it)
  float lg = 0.f, lb = 0.f;
  auto fetch_gb = [&](int c) {
    const int i = c * C + lane;
    const int64_t t = t0 + min(i, n - 1);
    lg = gb ? gb[t * 2 * D.H + h] : ld;
    lb = gb ? gb[(t * 2 + 1) * D.H + h] : 1.f;
    if (i >= n) lg = lb = 0.f;  // rows past the end neither decay nor add anything
  };
  auto scan_gb = [&](int c) {
    double G = (double)lg;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const double p = __shfl_up(G, o, 64);
      if (lane >= o) G += p;
    }
    const double GC = __shfl(G, 63, 64);
    const int b = (c & 1) * C + lane;
    Gs[b] = G;
    bs[b] = lb;
    eg[b] = expf((float)G);
    ws[b] = expf((float)(GC - G)) * lb;
  };
  fetch(0);
  if (w == 0) {
    fetch_gb(0);
    scan_gb(0);
  }
  for (int c = 0; c < nc; ++c) {
    const int cb = (c & 1) * C;
    stage(c);
    if (c + 1 < nc) {
      fetch(c + 1);
      if (w == (c & 3)) fetch_gb(c + 1);
    }
    lds_barrier();
    // ---- P, row tile w
    {
      bf16x8 qa[NK];
#pragma unroll
      for (int kk = 0; kk < NK; ++kk) qa[kk] = *reinterpret_cast<const bf16x8*>(Qs + (16 * w + l16) * KP + 32 * kk + 8 * q4);
      double gi[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) gi[r] = Gs[cb + 16 * w + 4 * q4 + r];
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        if (jt > (w | 1)) break;  // read-out takes pairs of tiles: above the diagonal only the pair's second one is read
        f32x4 s = {0.f, 0.f, 0.f, 0.f};
        if (jt <= w) {
#pragma unroll
          for (int kk = 0; kk < NK; ++kk)
            s = mfma(qa[kk], *reinterpret_cast<const bf16x8*>(Ks + (16 * jt + l16) * KP + 32 * kk + 8 * q4), s);
        }
        const int j = 16 * jt + l16;
        const double gj = Gs[cb + j];
        const float bj = bs[cb + j];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = 16 * w + 4 * q4 + r;
          const float x = j <= i ? s[r] * expf((float)(gi[r] - gj)) * bj : 0.f;
          bf16 a, b, d;
          split3(x, a, b, d);
          Ps[i * PP + j] = a;
          Ps[(C + i) * PP + j] = b;
          Ps[(2 * C + i) * PP + j] = d;
        }
      }
    }
    // ---- read-out of the state the chunk starts from: y^T [16 columns, 64 tokens] = S^T q^T
    f32x4 y[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) y[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      bf16x8 s0, s1, s2;  // k slot 8 q4 + e is key row 32 kk + 16 (e / 4) + 4 q4 + e % 4
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        bf16 a, b, d;
        split3(S[2 * kk + (e >> 2)][e & 3], a, b, d);
        s0[e] = a;
        s1[e] = b;
        s2[e] = d;
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const bf16* qr = Qs + (16 * i + l16) * KP + 32 * kk + 4 * q4;
        const bf16x4 lo = *reinterpret_cast<const bf16x4*>(qr), hi = *reinterpret_cast<const bf16x4*>(qr + 16);
        bf16x8 qb;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          qb[e] = lo[e];
          qb[4 + e] = hi[e];
        }
        y[i] = mfma(s2, qb, y[i]);
        y[i] = mfma(s1, qb, y[i]);
        y[i] = mfma(s0, qb, y[i]);
      }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) y[i] *= eg[cb + 16 * i + l16];
    // this wave's columns of v: lane l16 a column, tokens 32 s + 8 q4 + e
    bf16x8 vf[2];
#pragma unroll
    for (int s = 0; s < 2; ++s) vf[s] = read_tr(Vs, VP, 32 * s + 8 * q4, 32 * s + 8 * q4 + 4, 16 * w, l16);
    // ---- next state
    const float dc = eg[cb + C - 1];
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      bf16x8 u0, u1, u2;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        bf16 a, b, d;
        split3((float)vf[s][e] * ws[cb + 32 * s + 8 * q4 + e], a, b, d);
        u0[e] = a;
        u1[e] = b;
        u2[e] = d;
      }
#pragma unroll
      for (int t = 0; t < 2 * NK; ++t) {
        const bf16x8 kf = read_tr(Ks, KP, 32 * s + 8 * q4, 32 * s + 8 * q4 + 4, 16 * t, l16);
        if (s == 0) S[t] *= dc;
        S[t] = mfma(kf, u2, S[t]);
        S[t] = mfma(kf, u1, S[t]);
        S[t] = mfma(kf, u0, S[t]);
      }
    }
    lds_barrier();  // P is complete
    // ---- within the chunk
#pragma unroll
    for (int i = 0; i < 4; ++i) {
#pragma unroll
      for (int s = 0; s <= (i >> 1); ++s) {
        const bf16* pr = Ps + (16 * i + l16) * PP + 32 * s + 8 * q4;
        y[i] = mfma(vf[s], *reinterpret_cast<const bf16x8*>(pr + 2 * C * PP), y[i]);
        y[i] = mfma(vf[s], *reinterpret_cast<const bf16x8*>(pr + C * PP), y[i]);
        y[i] = mfma(vf[s], *reinterpret_cast<const bf16x8*>(pr), y[i]);
      }
      const int t = c * C + 16 * i + l16, cv = v0 + 16 * w + 4 * q4;
      const bf16x4 vv = *reinterpret_cast<const bf16x4*>(Vs + (16 * i + l16) * VP + 16 * w + 4 * q4);
      bf16x4 o;
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = (bf16)fmaf(sk, (float)vv[r], y[i][r]);
      if (t < n) {
        bf16* dst = out + ((int64_t)(t0 + t) * D.H + h) * D.dv + cv;
        if (cv + 3 < D.dv && D.dv % 4 == 0) {
          *reinterpret_cast<bf16x4*>(dst) = o;
        } else {
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (cv + r < D.dv) dst[r] = o[r];
        }
      }
    }
    if (c + 1 < nc && w == (c & 3)) scan_gb(c + 1);
    lds_barrier();
  }
  if (col < D.dv) {
#pragma unroll
    for (int t = 0; t < 2 * NK; ++t) {
      const int k = 16 * t + 4 * q4;
      if (k < dks) *reinterpret_cast<f32x4*>(st + k) = S[t];
    }
  }
  if (vt == 0 && D.taps > 1)
    advance_windows(conv_state + (int64_t)slots[seq] * (D.taps - 1) * D.channels, proj, t0, n, D, fresh, h);
}

template <int NK>
int launch(const void* qk, const void* v, const float* gb, const float* log_decay, const float* skip, const void* proj,
           float* state, void* conv_state, const int* seqs, int nseq, const int* cu, const int* start, const int* slots,
           void* out, const ScanDims& D, hipStream_t st) {
  constexpr int LDS = (2 * C * (32 * NK + 8) + C * VP + 3 * C * PP) * 2 + 2 * C * 8 + 6 * C * 4;
  static bool attr = false;
  if (!attr) {
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&decayed_chunk_kernel<NK>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, LDS);
    attr = true;
  }
  hipLaunchKernelGGL((decayed_chunk_kernel<NK>), dim3((unsigned)((D.dv + VT - 1) / VT * D.H * nseq)), dim3(NT), LDS, st,
                     (const bf16*)qk, (const bf16*)v, gb, log_decay, skip, (const bf16*)proj, state, (bf16*)conv_state, seqs,
                     cu, start, slots, (bf16*)out, D);
  DS_CHECK_LAUNCH();
  return 0;
}

}  // namespace

extern "C" int ds_scan_chunk_ok(int dk) { return dk <= 256; }

// bf16 storage, dk up to 256. seqs [nseq, 2]: (sequence, anything)
extern "C" int ds_scan_chunk(const void* qk, const void* v, const float* gb, const float* log_decay, const float* skip,
                             const void* proj, float* state, void* conv_state, const int* seqs, int nseq, const int* cu,
                             const int* start, const int* slots, void* out, const int* dims, int tokens, hipStream_t st) {
  if (nseq <= 0) return 0;
  const ScanDims D{dims[0], dims[1], dims[2], dims[3], dims[4], dims[5], dims[6], dims[7], dims[8], dims[9], dims[10], dims[11],
                   tokens};
  if (!scan_dims_ok(D) || !ds_scan_chunk_ok(D.dk) || (!gb == !log_decay) || (D.taps > 1 && !conv_state) ||
      (int64_t)nseq * D.H * ((D.dv + VT - 1) / VT) > INT32_MAX)
    return (int)hipErrorInvalidValue;
#define GO(NK)                                                                                                      \
  return launch<NK>(qk, v, gb, log_decay, skip, proj, state, conv_state, seqs, nseq, cu, start, slots, out, D, st)
  if (D.dk <= 32) GO(1);
  if (D.dk <= 64) GO(2);
  if (D.dk <= 128) GO(4);
  GO(8);
#undef GO
}
