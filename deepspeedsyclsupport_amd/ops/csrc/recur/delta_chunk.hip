// Gated delta rule over long portions, by chunks of 64 tokens (CDNA4, gfx950). See delta_rule.hip for the recurrence.
//
// With the running log decay G_i of a chunk (its first token included) and the state S0 the chunk starts from, unrolling
// the recurrence gives
//     (I + A) U = diag(beta) (V - diag(e^G) K S0),        A_ij = beta_i e^{G_i - G_j} (k_i . k_j),  j < i
//     o_i = e^{G_i} S0^T q_i + sum_{j <= i} P_ij u_j,      P_ij = e^{G_i - G_j} (q_i . k_j)
//     S   = e^{G_C} S0 + sum_j e^{G_C - G_j} k_j u_j^T
//  * chunk kernel: one workgroup per (chunk, head), all chunks of all sequences at once. K K^T and Q K^T on the fp32
//    matrix cores, then W = (I + A)^-1 diag(beta e^G) K and X = (I + A)^-1 diag(beta) V by forward substitution over
//    16-row blocks (the diagonal blocks inverted first), again products of 16 x 16 tiles. Writes W, X, P and the decays.
//  * scan kernel: one workgroup per (sequence, head, 16 value columns) walks the chunks: U = X - W S0, the read-out and
//    the next state are products of 16 x 16 tiles on the fp32 matrix cores; the state tile stays in LDS.
//  * norm kernel: per-head RMS norm and gate of the read-out.
// Everything is fp32: v_mfma_f32_16x16x4_f32 has the precision of the vector unit. The chunk borders are counted from
// the portion's first token; where they fall changes rounding only. Log decays are summed in fp64: only differences
// enter, and a strong decay early in a chunk must not cost the later ones their digits.
#include "delta_rule.h"

namespace {

constexpr int C = 64;
constexpr int NT = 256;

__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// Workgroup barrier for LDS: earlier LDS accesses have completed, global loads may still be under way
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// 4 consecutive elements of a row padded to d (a multiple of 4), zero beyond its end; one unconditional access
__device__ __forceinline__ f32x4 load4(const float* row, int k, int d) {
  const f32x4 v = *reinterpret_cast<const f32x4*>(row + min(k, d - 4));
  const float z = k < d ? 1.f : 0.f;
  return v * z;
}
// the same without the zeros, for products whose other operand has them: the value is not touched before its use
__device__ __forceinline__ f32x4 load4_raw(const float* row, int k, int d) {
  return *reinterpret_cast<const f32x4*>(row + min(k, d - 4));
}

// NK: 16-wide tiles of the key width (rounded up)
template <typename T, int NK>
__global__ void __launch_bounds__(NT) delta_chunk_kernel(
    const float* __restrict__ qk, const T* __restrict__ v, const float* __restrict__ gb, const int* __restrict__ cu,
    const int* __restrict__ work, float* __restrict__ Wo, float* __restrict__ Xo, float* __restrict__ Po,
    float* __restrict__ dec, DeltaDims D) {
  __shared__ __attribute__((aligned(16))) float A[C][C + 4];
  __shared__ double G[C];
  __shared__ float beta[C], eg[C];
  const int bid = xcd_remap(blockIdx.x, gridDim.x);  // the heads of a key group share its rows in one L2
  const int h = bid % D.H, ci = bid / D.H, hk = h / (D.H / D.Hk);
  const int seq = work[2 * ci], c = work[2 * ci + 1];
  const int t0 = cu[seq] + c * C, n = min(C, cu[seq + 1] - t0);
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, l16 = lane & 15, q4 = lane >> 4;
  const int64_t base = (int64_t)ci * D.H + h;
  if (w == 0) {
    double g = lane < n ? (double)gb[((int64_t)(t0 + lane) * 2) * D.H + h] : 0.0;
    for (int o = 1; o < 64; o <<= 1) {
      const double p = __shfl_up(g, o, 64);
      if (lane >= o) g += p;
    }
    G[lane] = g;
    beta[lane] = lane < n ? gb[((int64_t)(t0 + lane) * 2 + 1) * D.H + h] : 0.f;
    const double gc = __shfl(g, 63, 64);  // rows beyond n add nothing
    eg[lane] = expf((float)g);
    dec[base * 2 * C + lane] = eg[lane];
    dec[base * 2 * C + C + lane] = expf((float)(gc - g));
  }
  __syncthreads();
  // ---- K K^T and Q K^T, lower triangle of 16 x 16 tiles; wave w owns row tile w
  const int dks = D.dks();
  const float* kbase = qk + D.k_at(hk, 0);
  const float* qbase = qk + D.q_at(hk, 0);
  const int64_t rs = dks;
  const int64_t ri = (int64_t)(t0 + min(w * 16 + l16, n - 1)) * rs;
  f32x4 ka[NK], qa[NK];
#pragma unroll
  for (int t = 0; t < NK; ++t) {
    ka[t] = load4(kbase + ri, 16 * t + 4 * q4, dks);
    qa[t] = load4(qbase + ri, 16 * t + 4 * q4, dks);
  }
  for (int jt = 0; jt < 4; ++jt) {
    f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qq = {0.f, 0.f, 0.f, 0.f};
    if (jt <= w) {
      const int64_t rj = (int64_t)(t0 + min(jt * 16 + l16, n - 1)) * rs;
      f32x4 kb[NK];
#pragma unroll
      for (int t = 0; t < NK; ++t) kb[t] = load4(kbase + rj, 16 * t + 4 * q4, dks);
#pragma unroll
      for (int t = 0; t < NK; ++t)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          kk = mfma4(ka[t][e], kb[t][e], kk);
          qq = mfma4(qa[t][e], kb[t][e], qq);
        }
    }
    float* prow = Po + base * C * C;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = w * 16 + 4 * q4 + r, j = jt * 16 + l16;
      const float d = j <= i ? expf((float)(G[i] - G[j])) : 0.f;
      A[i][j] = j < i && i < n ? beta[i] * d * kk[r] : 0.f;
      prow[i * C + j] = j <= i && i < n ? d * qq[r] : 0.f;
    }
  }
  __syncthreads();
  // ---- invert the unit lower-triangular diagonal blocks, wave w block w, a column per lane
  if (lane < 16) {
    float t[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float r = i == lane ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) r = fmaf(-A[w * 16 + i][w * 16 + j], t[j], r);
      t[i] = r;
    }
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int i = 0; i < 16; ++i) A[w * 16 + i][w * 16 + lane] = t[i];
  }
  __syncthreads();
  // ---- block forward substitution of [W | X], 16 columns per wave at a time: x_b = T_bb (r_b - sum_{c < b} A_bc x_c).
  // A product's result layout (row 4 q4 + r of column l16) is the next one's right operand as it stands.
  const int wt = (dks + 15) / 16, xt = (D.dv + 15) / 16;
  for (int ct = w; ct < wt + xt; ct += 4) {
    const bool isw = ct < wt;
    const int col = (isw ? ct : ct - wt) * 16 + l16, width = isw ? dks : D.dv;
    const int cc = min(col, width - 1);
    f32x4 x[4];
#pragma unroll
    for (int b = 0; b < 4; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = b * 16 + 4 * q4 + r;
        const int64_t t = t0 + min(i, n - 1);
        // (rows past the end have beta 0, columns past it are not stored)
        if (isw) x[b][r] = kbase[t * rs + cc] * (beta[i] * eg[i]);
        else x[b][r] = (float)v[D.v_at(h, t) + cc] * beta[i];
      }
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int c2 = 0; c2 < b; ++c2) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(&A[b * 16 + l16][c2 * 16 + 4 * q4]);
#pragma unroll
        for (int e = 0; e < 4; ++e) acc = mfma4(a[e], x[c2][e], acc);
      }
      const f32x4 rhs = x[b] - acc, a = *reinterpret_cast<const f32x4*>(&A[b * 16 + l16][b * 16 + 4 * q4]);
      f32x4 y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int e = 0; e < 4; ++e) y = mfma4(a[e], rhs[e], y);
      x[b] = y;
    }
    if (col < width) {
      float* dst = (isw ? Wo + base * C * dks : Xo + base * C * D.dv) + col;
#pragma unroll
      for (int b = 0; b < 4; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) dst[(b * 16 + 4 * q4 + r) * width] = x[b][r];
    }
  }
}

template <typename T, int NK>
__global__ void __launch_bounds__(NT, (NK <= 8 ? 2 : 1)) delta_scan_kernel(
    const float* __restrict__ qk, const T* __restrict__ proj, const float* __restrict__ Wo, const float* __restrict__ Xo,
    const float* __restrict__ Po, const float* __restrict__ dec, const int* __restrict__ seqs, const int* __restrict__ cu,
    const int* __restrict__ start, const int* __restrict__ slots, float* __restrict__ state, T* __restrict__ conv_state,
    float* __restrict__ o, DeltaDims D) {
  constexpr int LD = 20;  // the four row groups of an operand read (4 rows apart) fall on different banks
  __shared__ float S[NK * 16][LD];
  __shared__ float U[C][LD];
  // the value tiles of a head walk the same W, P, q and k: neighbours in one XCD's L2
  const int bid = xcd_remap(blockIdx.x, gridDim.x), vts = (D.dv + 15) / 16;
  const int vt = bid % vts, h = bid / vts % D.H, sq = bid / (vts * D.H), seq = seqs[2 * sq], first = seqs[2 * sq + 1];
  const int hk = h / (D.H / D.Hk), tid = threadIdx.x, lane = tid & 63, w = tid >> 6, l16 = lane & 15, q4 = lane >> 4;
  const int t0 = cu[seq], n = cu[seq + 1] - t0, nc = (n + C - 1) / C, v0 = vt * 16;
  const bool fresh = start[seq] == 0;
  float* st = state + ((int64_t)slots[seq] * D.H + h) * D.dks() * D.dv;
  for (int i = tid; i < NK * 256; i += NT) {
    const int k = i % (NK * 16), j = i / (NK * 16);
    S[k][j] = (!fresh && k < D.dk && v0 + j < D.dv) ? st[(int64_t)(v0 + j) * D.dks() + k] : 0.f;
  }
  const int dks = D.dks();
  const int64_t rs = dks;
  const float* qbase = qk + D.q_at(hk, 0);
  const float* kbase = qk + D.k_at(hk, 0);
  const int vc = min(v0 + l16, D.dv - 1);  // columns past the end compute what nobody stores
  constexpr int KT = (NK + 3) / 4;  // key tiles of the state per wave
  f32x4 wf[NK], qf[NK], pf[4];
  float kf[KT][16], xf[4], dq[4], du[4], dc = 0.f;
  // The next chunk's operands are requested as soon as this chunk's are used up; the barriers below order LDS only, so
  // the requests stay in flight across them.
  const int row = w * 16 + l16, last = t0 + n - 1;
  auto fetch_rows = [&](int c) {
    const int64_t base = (int64_t)(first + c) * D.H + h;
    const float* wr = Wo + (base * C + row) * dks;
    const float* qr = qbase + (int64_t)min(t0 + c * C + row, last) * rs;
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      wf[kk] = load4_raw(wr, 16 * kk + 4 * q4, dks);  // rows of S past the key width stay zero
      qf[kk] = load4_raw(qr, 16 * kk + 4 * q4, dks);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = w * 16 + 4 * q4 + r;
      xf[r] = Xo[(base * C + i) * D.dv + vc];
      dq[r] = dec[base * 2 * C + i];
    }
  };
  auto fetch_p = [&](int c) {
    const int64_t base = (int64_t)(first + c) * D.H + h;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      du[r] = dec[base * 2 * C + C + w * 16 + 4 * q4 + r];
      pf[r] = *reinterpret_cast<const f32x4*>(Po + (base * C + row) * C + 16 * r + 4 * q4);
    }
  };
  auto fetch_keys = [&](int c) {
    const int tc = t0 + c * C;
    dc = dec[((int64_t)(first + c) * D.H + h) * 2 * C + C - 1];
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const int d = (w + 4 * kt) * 16 + l16;
#pragma unroll
      for (int i = 0; i < 16; ++i) {  // k index of the product: token 16 (i / 4) + 4 q4 + i % 4
        const int tok = min(tc + 16 * (i >> 2) + 4 * q4 + (i & 3), last);
        kf[kt][i] = kbase[(int64_t)tok * rs + min(d, dks - 1)];
      }
    }
  };
  fetch_rows(0);
  fetch_p(0);
  fetch_keys(0);
  lds_barrier();
  for (int c = 0; c < nc; ++c) {
    const int cn = min(c + 1, nc - 1);
    f32x4 u = {0.f, 0.f, 0.f, 0.f}, oq = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kk = 0; kk < NK; ++kk)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float s = S[16 * kk + 4 * q4 + e][l16];
        u = mfma4(wf[kk][e], s, u);
        oq = mfma4(qf[kk][e], s, oq);
      }
    f32x4 uu, acc;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      uu[r] = xf[r] - u[r];
      acc[r] = dq[r] * oq[r];
      U[w * 16 + 4 * q4 + r][l16] = uu[r];
    }
    fetch_rows(cn);
    lds_barrier();
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
      if (jt > w) break;  // P is lower triangular
#pragma unroll
      for (int e = 0; e < 4; ++e) acc = mfma4(pf[jt][e], U[16 * jt + 4 * q4 + e][l16], acc);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = c * C + w * 16 + 4 * q4 + r;
      if (i < n && v0 + l16 < D.dv) o[D.v_at(h, t0 + i) + v0 + l16] = acc[r];
    }
    lds_barrier();
    // U <- e^{G_C - G_i} U for the state update (every wave its own rows)
#pragma unroll
    for (int r = 0; r < 4; ++r) U[w * 16 + 4 * q4 + r][l16] = uu[r] * du[r];
    fetch_p(cn);
    lds_barrier();
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const int d0 = (w + 4 * kt) * 16;
      if (w + 4 * kt < NK) {
        f32x4 s;
#pragma unroll
        for (int r = 0; r < 4; ++r) s[r] = dc * S[d0 + 4 * q4 + r][l16];
#pragma unroll
        for (int i = 0; i < 16; ++i) s = mfma4(kf[kt][i], U[16 * (i >> 2) + 4 * q4 + (i & 3)][l16], s);
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (d0 + 4 * q4 < dks) S[d0 + 4 * q4 + r][l16] = s[r];
      }
    }
    fetch_keys(cn);
    lds_barrier();
  }
  for (int i = tid; i < NK * 256; i += NT) {
    const int k = i % (NK * 16), j = i / (NK * 16);
    if (k < D.dk && v0 + j < D.dv) st[(int64_t)(v0 + j) * D.dks() + k] = S[k][j];
  }
  if (vt == 0 && D.taps > 1)
    advance_head(conv_state + (int64_t)slots[seq] * (D.taps - 1) * D.channels(), proj, t0, n, D, fresh, h);
}

// out = o / rms(o) * w * silu(gate), one wave per (token, head) of the long sequences' chunks
template <typename T, bool PAIR>
__global__ void __launch_bounds__(NT) delta_norm_kernel(const float* __restrict__ o, const T* __restrict__ proj,
                                                        const float* __restrict__ norm_w, float eps,
                                                        const int* __restrict__ cu, const int* __restrict__ work,
                                                        T* __restrict__ out, DeltaDims D) {
  const int h = blockIdx.x % D.H, ci = blockIdx.x / D.H, lane = threadIdx.x & 63;
  const int seq = work[2 * ci], t0 = cu[seq] + work[2 * ci + 1] * C, n = min(C, cu[seq + 1] - t0);
  float nw[2][2];
#pragma unroll
  for (int k = 0; k < 2; ++k) load2<PAIR>(norm_w, k * 128 + 2 * lane, D.dv, nw[k]);
  constexpr int UNR = 4;
  for (int i0 = threadIdx.x >> 6; i0 < n; i0 += UNR * NT / 64) {
    float x[UNR][2][2], g[UNR][2][2];
#pragma unroll
    for (int u = 0; u < UNR; ++u) {
      const int64_t t = t0 + min(i0 + u * (NT / 64), n - 1);
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        x[u][k][0] = x[u][k][1] = 0.f;
        if (k * 128 >= D.dv) continue;
        const int c = k * 128 + 2 * lane;
        load2<PAIR>(o + D.v_at(h, t), c, D.dv, x[u][k]);
        load2<PAIR>(proj + t * D.row() + D.channels() + h * D.dv, c, D.dv, g[u][k]);
        x[u][k][0] *= c < D.dv ? 1.f : 0.f;
        x[u][k][1] *= c + 1 < D.dv ? 1.f : 0.f;
      }
    }
#pragma unroll
    for (int u = 0; u < UNR; ++u) {
      const int i = i0 + u * (NT / 64);
      if (i >= n) break;
      float ss = 0.f;
#pragma unroll
      for (int k = 0; k < 2; ++k) ss = fmaf(x[u][k][0], x[u][k][0], fmaf(x[u][k][1], x[u][k][1], ss));
      const float rms = 1.f / sqrtf(wave_sum(ss) / (float)D.dv + eps);
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        if (k * 128 >= D.dv) continue;
#pragma unroll
        for (int e = 0; e < 2; ++e) g[u][k][e] = x[u][k][e] * rms * nw[k][e] * silu(g[u][k][e]);
        store2<PAIR>(out + ((int64_t)(t0 + i) * D.H + h) * D.dv, k * 128 + 2 * lane, D.dv, g[u][k]);
      }
    }
  }
}

template <typename T>
int run(const float* qk, const void* v, const float* gb, const void* proj, const float* norm_w, float eps, float* state,
        void* conv_state, const int* seqs, int nseq, const int* work, int nwork, const int* cu, const int* start,
        const int* slots, float* ws, float* o, void* out, DeltaDims D, hipStream_t st) {
  float* W = ws;
  float* X = W + (int64_t)nwork * D.H * C * D.dks();
  float* P = X + (int64_t)nwork * D.H * C * D.dv;
  float* dec = P + (int64_t)nwork * D.H * C * C;
  const dim3 grid((unsigned)((D.dv + 15) / 16 * D.H * nseq));
#define GO(NK)                                                                                                       \
  {                                                                                                                  \
    hipLaunchKernelGGL((delta_chunk_kernel<T, NK>), dim3(nwork * D.H), dim3(NT), 0, st, qk, (const T*)v, gb, cu, work, \
                       W, X, P, dec, D);                                                                             \
    DS_CHECK_LAUNCH();                                                                                               \
    hipLaunchKernelGGL((delta_scan_kernel<T, NK>), grid, dim3(NT), 0, st, qk, (const T*)proj, W, X, P, dec, seqs, cu,  \
                       start, slots, state, (T*)conv_state, o, D);                                                   \
  }
  if (D.dk <= 32) GO(2)
  else if (D.dk <= 64) GO(4)
  else if (D.dk <= 128) GO(8)
  else GO(16)
#undef GO
  DS_CHECK_LAUNCH();
#define NORM(PAIR)                                                                                                   \
  hipLaunchKernelGGL((delta_norm_kernel<T, PAIR>), dim3(nwork * D.H), dim3(NT), 0, st, o, (const T*)proj, norm_w, eps, \
                     cu, work, (T*)out, D)
  if (D.dv % 2 == 0 && D.dk % 2 == 0) NORM(true);
  else NORM(false);
#undef NORM
  DS_CHECK_LAUNCH();
  return 0;
}

}  // namespace

// fp32 words of workspace a call needs
extern "C" int64_t ds_delta_chunk_ws(int nwork, int H, int dk, int dv) {
  return (int64_t)nwork * H * C * ((dk + 3) / 4 * 4 + dv + C + 2);
}

// seqs [nseq, 2]: (sequence, index of its first entry in work); work [nwork, 2]: (sequence, chunk), a sequence's chunks
// in order. o: fp32 [H, tokens, dv] scratch.
extern "C" int ds_delta_chunk(const float* qk, const void* v, const float* gb, const void* proj, const float* norm_w,
                              float eps, float* state, void* conv_state, const int* seqs, int nseq, const int* work,
                              int nwork, const int* cu, const int* start, const int* slots, float* ws, float* o,
                              void* out, int tokens, int Hk, int H, int dk, int dv, int taps, int dtype,
                              hipStream_t st) {
  if (nseq <= 0 || nwork <= 0) return 0;
  const DeltaDims D{Hk, H, dk, dv, taps, tokens};
  if (!dims_ok(D) || (int64_t)nwork * H * 16 > INT32_MAX) return (int)hipErrorInvalidValue;
  if (dtype == DS_F32)
    return run<float>(qk, v, gb, proj, norm_w, eps, state, conv_state, seqs, nseq, work, nwork, cu, start, slots, ws, o,
                      out, D, st);
  if (dtype == DS_BF16)
    return run<bf16>(qk, v, gb, proj, norm_w, eps, state, conv_state, seqs, nseq, work, nwork, cu, start, slots, ws, o, out,
                     D, st);
  return (int)hipErrorInvalidValue;
}
