// Ragged paged flash attention for inference prefill / prompt chunks (SplitFuse), bf16, head dims 64 / 80 / 96 / 128 /
// 256 (GPT-2 / Phi / GPT-NeoX-20B / Llama / GPT-J).
//
// Reference counterpart (behaviour): inference v2's `blocked_flash` (`inference/v2/kernels/ragged_ops/blocked_flash/
// blocked_flash.cpp:21-100`, a prebuilt flash-attention over the blocked KV cache driven by the ragged batch's
// `atoms`) and v1's `softmax_context` with ALiBi / local windows (`csrc/transformer/inference/csrc/softmax.cu:35,256`).
//
// One launch covers every prompt / chunk sequence of a ragged batch:
//  * queries are the batch's concatenated new tokens q [T, Hq, D] (cu_q gives each sequence's slice); keys and
//    values are read straight from the paged cache [blocks, Hk, BS, D] through the block table — the new tokens'
//    K/V were appended by the fused QKV epilogue first, so a chunk sees its whole cached prefix plus itself;
//  * a host-built work list names (sequence, 128-row query block) pairs, so ragged lengths cost no padding beyond one
//    block; every q head of a work item sits on one XCD (xcd_remap) so the GQA group's K/V tiles are shared in L2;
//  * per query row the position is start + i: causal masking against absolute positions, ALiBi bias
//    slope_h * (key - pos) folded into the score before the online softmax, sliding window key > pos - window; tiles
//    entirely outside [pos - window, pos] are never loaded;
//  * the compute core is flash_fwd.hip's: 4 waves x 32 rows, S^T = K.Q^T on v_mfma_f32_32x32x16_bf16 so each lane
//    owns one query row's scores, P reused as the A operand of O += P.V, V by ds_read_b64_tr_b16 from the same
//    XOR-swizzled LDS image, next tile's loads issued before the current tile's MFMAs;
//  * a second instantiation (EXT) takes key and value widths of their own (any multiple of 8, tiled at the next of 32 /
//    64 / 128 / 256), chunked visibility (key >= pos - pos % chunk) and a tanh score cap, with their sizes as run-time
//    arguments. It keeps the softmax weights to 16 mantissa bits through the P.V product (two bf16 operands, high + low);
//  * a third (LATENT) reads keys and values that were expanded from cached latents: rows laid end to end, a sequence's from
//    kv_offs on, [keys of all heads | values of all heads] per row, with the last key columns (one rotated part for all
//    heads) in the latent's own row. Its workgroups go head by head, so an XCD's L2 serves one head's keys;
//  * EXT and LATENT take a softmax sink per head: exp(sink) joins the denominator; EXT a gate per token and head: the output
//    times its sigmoid;
//  * the head dim is a template parameter: D / 16 MFMA steps for the scores, ceil(D / 32) output column tiles (D = 80
//    computes a third, half-used tile over zero-filled LDS columns), LDS rows pitched to 16 (D <= 128) or 32 (D = 256)
//    16-byte chunks so one swizzle serves every size.
#pragma once
#include "ds_hip.h"

namespace {

enum : int { PLAIN = 0, EXT_ = 1, LATENT = 2 };
constexpr int BM = 128;
constexpr int BN = 64;
constexpr int NTHR = 256;

template <int DK, int DV>
struct Cfg {
  static_assert(DK % 16 == 0 && DK >= 32 && DK <= 256 && DV % 16 == 0 && DV >= 32 && DV <= 256, "head dims");
  static constexpr int KC = DK / 16;               // MFMA steps of the score product
  static constexpr int DT = (DV + 31) / 32;        // 32-column output tiles
  static constexpr int PK = DK <= 128 ? 16 : 32;   // 16-byte chunks per LDS row (pitch) of K, V
  static constexpr int PV = DV <= 128 ? 16 : 32;
  static constexpr int KBYTES = BN * PK * 16;
  static constexpr int VBYTES = BN * PV * 16;
  static constexpr int NLK = BN * PK / NTHR;       // chunks staged per thread per tile
  static constexpr int NLV = BN * PV / NTHR;
  static constexpr int LDS_BYTES = 2 * KBYTES + 2 * VBYTES + 4 * 32 * 4;
  static constexpr int OCC = DK <= 128 && DV <= 128 ? 2 : 1;
};

typedef short s16x4_t __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x16_t __attribute__((ext_vector_type(16)));
typedef unsigned int u32x4_t __attribute__((ext_vector_type(4)));

template <int ROWB>
__device__ __forceinline__ int lds_off(int row, int ch) {
  return row * ROWB + 16 * (ch ^ (((row & 3) << 2) | ((row >> 2) & 3)));
}

struct PagedArgs {
  const bf16* q;          // [T, Hq, D], ldq elements from row to row
  const bf16* kc;         // [blocks, Hk, BS, D]
  const bf16* vc;
  bf16* o;                // [T, Hq, D], ldo elements from row to row
  const int* block_table; // [nseq, max_blocks]
  const int* start;       // [nseq] cached tokens before this step
  const int* cu_q;        // [nseq + 1] token offsets of each sequence's new tokens
  const int* work;        // [nwork, 2] (sequence, query block)
  const float* alibi;     // [Hq] slopes or null
  int Hq, Hk, BS, max_blocks, window;
  float c;                // softmax scale * log2(e)
  float inv_scale;        // 1 / softmax scale (ALiBi bias in score units)
  int dk, dv, chunk;      // EXT: head widths, chunk of the visibility mask (0: none)
  const float* sink;      // EXT, LATENT: [Hq] or null
  const int* kv_offs;     // LATENT: first context row of sequence `first`, and of the ones after it
  int first, dn, ldk, ldr, rot0;  // key columns of a head (the rest is rotated), row lengths of kc and of vc, first rotated
                          // column there; kc: the expanded rows, vc: the latents' rows
  const int* kv_first;    // LATENT: first key of those contexts (whole tiles into the sequence), or null: 0
  int64_t ldo, ldq;       // elements from a token's row of o / q to the next one's
  const bf16* gate;       // EXT: [T, Hq], ldg elements from row to row, or null
  int64_t ldg;
  float cap_in, cap_out;  // EXT: capped score in log2 units = cap_out * tanh(score * cap_in); cap_out 0: no cap
};

template <int DK, int DV, int MODE>
__global__ void __launch_bounds__(NTHR, (Cfg<DK, DV>::OCC)) paged_prefill_kernel(PagedArgs a) {
  using C = Cfg<DK, DV>;
  constexpr bool EXT = MODE != PLAIN, LAT = MODE == LATENT;
  constexpr int KC = C::KC, DT = C::DT, PK = C::PK, PV = C::PV, RK = PK * 16, RV = PV * 16, NLK = C::NLK, NLV = C::NLV;
  const int dk = EXT ? a.dk : DK, dv = EXT ? a.dv : DV;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6, h = lane >> 5, l32 = lane & 31;
  const int logical = xcd_remap(blockIdx.x, gridDim.x);
  const int per_head = gridDim.x / a.Hq;
  // (LATENT: the longest rows of a head first, they are the last of the work list)
  const int w = LAT ? per_head - 1 - logical % per_head : logical / a.Hq;
  const int hq = LAT ? logical / per_head : logical % a.Hq, hk = hq / (a.Hq / a.Hk);
  const int seq = a.work[2 * w], qb = a.work[2 * w + 1];
  const int t0 = a.cu_q[seq], n = a.cu_q[seq + 1] - t0, start = a.start[seq], Skv = start + n;
  const int q0 = qb * BM, q0w = q0 + wid * 32;
  const int* bt = LAT ? nullptr : a.block_table + (int64_t)seq * a.max_blocks;
  // (LATENT: the row of key 0, were it there)
  const int64_t ctx0 = LAT ? a.kv_offs[seq - a.first] - (a.kv_first ? a.kv_first[seq - a.first] : 0) : 0;
  const float slope = a.alibi ? a.alibi[hq] * a.inv_scale : 0.f;

  bf16x8_t qf[KC];
  {
    const int qr = min(q0w + l32, n - 1);
    const bf16* qrow = a.q + (int64_t)(t0 + qr) * a.ldq + hq * dk + 8 * h;
#pragma unroll
    for (int kk = 0; kk < KC; ++kk) {
      if (!EXT || 16 * kk + 8 * h < dk) {
        qf[kk] = *reinterpret_cast<const bf16x8_t*>(qrow + 16 * kk);
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) qf[kk][e] = (bf16)0.f;
      }
    }
  }
  const int pos_lane = start + q0w + l32;                // this lane's query position
  const int pos_hi = start + min(q0 + BM, n) - 1;        // last query position of the block
  const int wpos_lo = start + q0w, wpos_hi = start + q0w + 31;
  int kt1 = min((Skv + BN - 1) / BN, pos_hi / BN + 1);
  // first key a position sees (non-decreasing in the position)
  auto first_key = [&](int p) {
    int lo = MODE == EXT_ && a.chunk > 0 ? p / a.chunk * a.chunk : 0;
    if (a.window > 0) lo = max(lo, p - a.window + 1);
    return lo;
  };
  const int lo_lane = first_key(pos_lane), lo_whi = first_key(wpos_hi), lo_wlo = first_key(wpos_lo);
  int kt0 = first_key(start + q0) / BN;
  if (kt0 > kt1) kt0 = kt1;

  char* const ksm = smem;
  char* const vsm = smem + 2 * C::KBYTES;
  float* scratch = reinterpret_cast<float*>(smem + 2 * C::KBYTES + 2 * C::VBYTES) + wid * 32;
  constexpr int CK = LAT ? DK / 8 : PK, CV = LAT ? DV / 8 : PV;    // pieces of a row that are staged
  constexpr int NK_ = LAT ? BN * CK / NTHR : NLK, NV_ = LAT ? BN * CV / NTHR : NLV;
  u32x4_t kreg[NK_], vreg[NV_];
  // LATENT: rows lie end to end, so every piece has a place of its own that moves on by the same step with every tile. Pieces
  // past the widths repeat the last one: there the queries are zero, or nothing is stored. (Rows past the context's end are
  // masked; 64 of them exist behind the last context.)
  const bf16* kp_[NK_];
  const bf16* vp_[NV_];
  int kstep[NK_];
  if constexpr (LAT) {
#pragma unroll
    for (int i = 0; i < NK_; ++i) {
      const int row = (tid + i * NTHR) / CK, c = min((tid + i * NTHR) % CK * 8, dk - 8);
      const bool up = c < a.dn;
      const int64_t r_ = ctx0 + (int64_t)kt0 * BN + row;
      kp_[i] = up ? a.kc + r_ * a.ldk + hq * a.dn + c : a.vc + r_ * a.ldr + a.rot0 + c - a.dn;
      kstep[i] = BN * (up ? a.ldk : a.ldr);
    }
#pragma unroll
    for (int i = 0; i < NV_; ++i) {
      const int row = (tid + i * NTHR) / CV, c = min((tid + i * NTHR) % CV * 8, dv - 8);
      vp_[i] = a.kc + (ctx0 + (int64_t)kt0 * BN + row) * a.ldk + a.Hq * a.dn + hq * dv + c;
    }
  }
  auto slot_of = [&](int tile, int row) {
    const int key = min(tile * BN + row, Skv - 1);
    return ((int64_t)bt[key / a.BS] * a.Hk + hk) * a.BS + key % a.BS;
  };
  auto stage_load = [&](int tile) {
    if constexpr (!EXT) {  // one pitch, one width: the key and value chunk share their address
#pragma unroll
      for (int i = 0; i < NLK; ++i) {
        const int cidx = tid + i * NTHR, row = cidx / PK, ch = cidx % PK;
        if (ch < DK / 8) {
          const int64_t off = slot_of(tile, row) * DK + ch * 8;
          kreg[i] = *reinterpret_cast<const u32x4_t*>(a.kc + off);
          vreg[i] = *reinterpret_cast<const u32x4_t*>(a.vc + off);
        } else {  // pitch padding: zero columns (read by the last, partly used output tile of D = 80)
          kreg[i] = u32x4_t{0u, 0u, 0u, 0u};
          vreg[i] = u32x4_t{0u, 0u, 0u, 0u};
        }
      }
    } else if constexpr (LAT) {  // tiles are asked for in order
#pragma unroll
      for (int i = 0; i < NK_; ++i) {
        kreg[i] = *reinterpret_cast<const u32x4_t*>(kp_[i]);
        kp_[i] += kstep[i];
      }
#pragma unroll
      for (int i = 0; i < NV_; ++i) {
        vreg[i] = *reinterpret_cast<const u32x4_t*>(vp_[i]);
        vp_[i] += BN * a.ldk;
      }
    } else {
#pragma unroll
      for (int i = 0; i < NLK; ++i) {
        const int cidx = tid + i * NTHR, row = cidx / PK, ch = cidx % PK;
        kreg[i] = u32x4_t{0u, 0u, 0u, 0u};
        if (ch * 8 < dk) kreg[i] = *reinterpret_cast<const u32x4_t*>(a.kc + slot_of(tile, row) * dk + ch * 8);
      }
#pragma unroll
      for (int i = 0; i < NLV; ++i) {
        const int cidx = tid + i * NTHR, row = cidx / PV, ch = cidx % PV;
        vreg[i] = u32x4_t{0u, 0u, 0u, 0u};
        if (ch * 8 < dv) vreg[i] = *reinterpret_cast<const u32x4_t*>(a.vc + slot_of(tile, row) * dv + ch * 8);
      }
    }
  };
  auto stage_store = [&](int buf) {
#pragma unroll
    for (int i = 0; i < NK_; ++i) {
      const int cidx = tid + i * NTHR, row = cidx / CK, ch = cidx % CK;
      if (LAT || ch < DK / 8) *reinterpret_cast<u32x4_t*>(ksm + buf * C::KBYTES + lds_off<RK>(row, ch)) = kreg[i];
    }
#pragma unroll
    for (int i = 0; i < NV_; ++i) {
      const int cidx = tid + i * NTHR, row = cidx / CV, ch = cidx % CV;
      if (LAT || ch < 4 * DT) *reinterpret_cast<u32x4_t*>(vsm + buf * C::VBYTES + lds_off<RV>(row, ch)) = vreg[i];
    }
  };

  f32x16_t o[DT];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[dt][r] = 0.f;
  float m_run = -INFINITY, l_run = 0.f;

  if (kt1 > kt0) {
    stage_load(kt0);
    stage_store(0);
  }
  __syncthreads();
  for (int j = kt0; j < kt1; ++j) {
    const int cur = (j - kt0) & 1;
    if (j + 1 < kt1) stage_load(j + 1);
    const int k0 = j * BN;
    const bool active = q0w < n && k0 <= wpos_hi && k0 + BN - 1 >= lo_wlo;
    if (active) {
      const char* Kt = ksm + cur * C::KBYTES;
      const char* Vt = vsm + cur * C::VBYTES;
      f32x16_t s[2];
#pragma unroll
      for (int t = 0; t < 2; ++t) {
#pragma unroll
        for (int r = 0; r < 16; ++r) s[t][r] = 0.f;
#pragma unroll
        for (int kk = 0; kk < KC; ++kk) {
          const bf16x8_t av = *reinterpret_cast<const bf16x8_t*>(Kt + lds_off<RK>(t * 32 + l32, 2 * kk + h));
          s[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(av, qf[kk], s[t], 0, 0, 0);
        }
      }
      // ALiBi bias, causal diagonal, window, key tail (lane = one query row, r = 32 keys of the 64)
      const bool need_mask = k0 + BN - 1 > wpos_lo || k0 < lo_whi || (!LAT && k0 + BN > Skv);
      if constexpr (MODE == EXT_) {
        if (a.cap_out > 0.f) {
#pragma unroll
          for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int r = 0; r < 16; ++r)  // tanh z = 1 - 2 / (e^2z + 1); cap_in carries the 2 log2(e)
              s[t][r] = a.cap_out * (1.f - 2.f * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s[t][r] * a.cap_in) + 1.f));
        }
      }
      if ((!LAT && a.alibi) || need_mask) {
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int key = k0 + t * 32 + (r & 3) + 8 * (r >> 2) + 4 * h;
            float v = LAT ? s[t][r] : fmaf(slope, (float)(key - pos_lane), s[t][r]);
            if ((!LAT && key >= Skv) || key > pos_lane || key < lo_lane) v = -INFINITY;
            s[t][r] = v;
          }
      }
      // a moderate cap bounds the scores: it serves as the maximum, and nothing is ever rescaled
      const bool fixed = MODE == EXT_ && a.cap_out > 0.f && a.cap_out <= 48.f;
      float alpha = 1.f, mc = a.cap_out;
      if (!fixed) {
        float mx = -INFINITY;
#pragma unroll
        for (int r = 0; r < 16; ++r) mx = fmaxf(mx, fmaxf(s[0][r], s[1][r]));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        const float m_new = fmaxf(m_run, mx);
        const float m_use = m_new == -INFINITY ? 0.f : m_new;
        alpha = __builtin_amdgcn_exp2f((m_run - m_use) * a.c);
        mc = m_use * a.c;
        m_run = m_new;
      }
      float psum = 0.f;
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const float p = __builtin_amdgcn_exp2f(fmaf(s[t][r], a.c, -mc));
          s[t][r] = p;
          psum += p;
        }
      l_run = l_run * alpha + psum;
      if (!fixed && !__all(alpha == 1.f)) {
        if (lane < 32) scratch[lane] = alpha;
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
        float a4[16];
#pragma unroll
        for (int g = 0; g < 4; ++g) {
          const f32x4 v = *reinterpret_cast<const f32x4*>(scratch + 8 * g + 4 * h);
#pragma unroll
          for (int i = 0; i < 4; ++i) a4[4 * g + i] = v[i];
        }
#pragma unroll
        for (int dt = 0; dt < DT; ++dt)
#pragma unroll
          for (int r = 0; r < 16; ++r) o[dt][r] *= a4[r];
        __builtin_amdgcn_wave_barrier();
      }
      const int gq = (lane >> 2) & 3, gch = (lane >> 1) & 1, gb = 8 * (lane & 1), colhalf = (lane >> 4) & 1;
      auto v_of = [&](int t, int ss, int dt) {  // 16 keys of 32 value columns, transposed on the way out of LDS
        const int ch0 = dt * 4 + colhalf * 2 + gch, rb = t * 32 + 16 * ss + 4 * h;
        const s16x4_t lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (__attribute__((address_space(3))) s16x4_t*)(Vt + lds_off<RV>(rb + gq, ch0) + gb));
        const s16x4_t hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (__attribute__((address_space(3))) s16x4_t*)(Vt + lds_off<RV>(rb + 8 + gq, ch0) + gb));
        s16x8 vv;
#pragma unroll
        for (int e = 0; e < 4; ++e) { vv[e] = lo[e]; vv[4 + e] = hi[e]; }
        return __builtin_bit_cast(bf16x8_t, vv);
      };
      // EXT, LATENT: weights as two bf16 terms, the second what the first leaves out
      if constexpr (LAT) {  // (16 keys at a time: with wide keys the registers are short)
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
          for (int ss = 0; ss < 2; ++ss) {
            bf16x8_t pa, pl;
#pragma unroll
            for (int e = 0; e < 8; ++e) {
              pa[e] = (bf16)s[t][8 * ss + e];
              pl[e] = (bf16)(s[t][8 * ss + e] - (float)pa[e]);
            }
#pragma unroll
            for (int dt = 0; dt < DT; ++dt) {
              const bf16x8_t vv = v_of(t, ss, dt);
              o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pa, vv, o[dt], 0, 0, 0);
              o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pl, vv, o[dt], 0, 0, 0);
            }
          }
      } else {
        bf16x8_t pa[2][2];
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
          for (int ss = 0; ss < 2; ++ss)
#pragma unroll
            for (int e = 0; e < 8; ++e) pa[t][ss][e] = (bf16)s[t][8 * ss + e];
        bf16x8_t pl[2][2];
        if constexpr (EXT) {
#pragma unroll
          for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int ss = 0; ss < 2; ++ss)
#pragma unroll
              for (int e = 0; e < 8; ++e) pl[t][ss][e] = (bf16)(s[t][8 * ss + e] - (float)pa[t][ss][e]);
        }
#pragma unroll
        for (int dt = 0; dt < DT; ++dt)
#pragma unroll
          for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int ss = 0; ss < 2; ++ss) {
              const bf16x8_t vv = v_of(t, ss, dt);
              o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pa[t][ss], vv, o[dt], 0, 0, 0);
              if constexpr (EXT) o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pl[t][ss], vv, o[dt], 0, 0, 0);
            }
      }
    }
    if (j + 1 < kt1) stage_store(cur ^ 1);
    __syncthreads();
  }

  const float l_tot = l_run + __shfl_xor(l_run, 32, 64);
  float inv = l_tot > 0.f ? 1.f / l_tot : 0.f;
  if constexpr (EXT) {
    if (a.sink) {  // in the frame of the maximum the weights were taken in
      const float sk = a.sink[hq] * 1.4426950408889634f, m = MODE == EXT_ && a.cap_out > 0.f && a.cap_out <= 48.f ? a.cap_out : m_run * a.c;
      const float mn = fmaxf(m, sk), f = __builtin_amdgcn_exp2f(m - mn);
      inv = f / fmaf(l_tot, f, __builtin_amdgcn_exp2f(sk - mn));
    }
  }
  if constexpr (MODE == EXT_) {
    if (a.gate) inv /= 1.f + __expf(-(float)a.gate[(int64_t)(t0 + min(q0w + l32, n - 1)) * a.ldg + hq]);
  }
  if (lane < 32) scratch[lane] = inv;
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  float iv[16];
#pragma unroll
  for (int g = 0; g < 4; ++g) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(scratch + 8 * g + 4 * h);
#pragma unroll
    for (int i = 0; i < 4; ++i) iv[4 * g + i] = v[i];
  }
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    const int qi = q0w + (r & 3) + 8 * (r >> 2) + 4 * h;
    if (qi < n) {
      bf16* orow = a.o + (int64_t)(t0 + qi) * a.ldo + hq * dv + l32;
#pragma unroll
      for (int dt = 0; dt < DT; ++dt)
        if ((!EXT && DV % 32 == 0) || dt * 32 + l32 < dv) orow[dt * 32] = (bf16)(o[dt][r] * iv[r]);
    }
  }
}

template <int DK, int DV, int MODE>
int launch(const PagedArgs& a, int nwork, hipStream_t st) {
  constexpr int LDS = Cfg<DK, DV>::LDS_BYTES;
  static bool attr = false;
  if (!attr) {
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&paged_prefill_kernel<DK, DV, MODE>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, LDS);
    attr = true;
  }
  hipLaunchKernelGGL((paged_prefill_kernel<DK, DV, MODE>), dim3(nwork * a.Hq), dim3(NTHR), LDS, st, a);
  DS_CHECK_LAUNCH();
  return 0;
}

}  // namespace
