// Ragged paged flash attention for inference prefill / prompt chunks (SplitFuse): entry points. The kernel is in
// paged_prefill_core.h.
#include "paged_prefill_core.h"

// q / o [T, Hq, D] bf16 (contiguous), caches [blocks, Hk, BS, D] bf16, D in {64, 80, 96, 128, 256}, block_table
// [nseq, max_blocks] int32, start [nseq], cu_q [nseq + 1], work [nwork, 2] (sequence, 128-row query block) int32,
// alibi [Hq] fp32 or null, window <= 0 for none.
extern "C" int ds_paged_prefill(const void* q, const void* kc, const void* vc, void* o, const int* block_table,
                                const int* start, const int* cu_q, const int* work, int nwork, const float* alibi,
                                int Hq, int Hk, int D, int BS, int max_blocks, int window, float scale,
                                hipStream_t st) {
  if (nwork <= 0) return 0;
  if (Hk <= 0 || Hq % Hk || BS <= 0 || max_blocks <= 0 || scale <= 0.f) return (int)hipErrorInvalidValue;
  PagedArgs a{(const bf16*)q, (const bf16*)kc, (const bf16*)vc, (bf16*)o, block_table, start, cu_q, work, alibi,
              Hq, Hk, BS, max_blocks, window, scale * 1.4426950408889634f, 1.f / scale, D, D, 0, nullptr, nullptr, 0, 0, 0, 0, 0, nullptr, (int64_t)Hq * D,
              (int64_t)Hq * D, nullptr, 0, 0.f, 0.f};
  switch (D) {
    case 64: return launch<64, 64, PLAIN>(a, nwork, st);
    case 80: return launch<80, 80, PLAIN>(a, nwork, st);
    case 96: return launch<96, 96, PLAIN>(a, nwork, st);
    case 128: return launch<128, 128, PLAIN>(a, nwork, st);
    case 256: return launch<256, 256, PLAIN>(a, nwork, st);
    default: return (int)hipErrorInvalidValue;
  }
}

// Key width dk and value width dv (multiples of 8 up to 256) of their own, chunked and / or windowed visibility,
// optional score cap: score = softcap * tanh(scale * q.k / softcap). sink [Hq] or null: exp(sink) joins the softmax's
// denominator. gate [T, Hq] or null: heads come out times its sigmoid. ldo, ldg: elements between the rows of o and gate.
extern "C" int ds_paged_prefill_ext(const void* q, const void* kc, const void* vc, void* o, const int* block_table,
                                    const int* start, const int* cu_q, const int* work, int nwork, int Hq, int Hk, int dk,
                                    int dv, int BS, int max_blocks, int window, int chunk, float scale, float softcap,
                                    const float* sink, const void* gate, int64_t ldg, int64_t ldo, hipStream_t st) {
  if (nwork <= 0) return 0;
  if (Hk <= 0 || Hq % Hk || BS <= 0 || max_blocks <= 0 || scale <= 0.f || dk % 8 || dv % 8 || dk <= 0 || dv <= 0 ||
      ldo < (int64_t)Hq * dv)
    return (int)hipErrorInvalidValue;
  constexpr float LOG2E = 1.4426950408889634f;
  const bool cap = softcap > 0.f;
  // with a cap the scores leave the capping step in log2 units already
  PagedArgs a{(const bf16*)q, (const bf16*)kc, (const bf16*)vc, (bf16*)o, block_table, start, cu_q, work, nullptr,
              Hq, Hk, BS, max_blocks, window, cap ? 1.f : scale * LOG2E, 1.f / scale, dk, dv, chunk,
              sink, nullptr, 0, 0, 0, 0, 0, nullptr, ldo, (int64_t)Hq * dk, (const bf16*)gate, ldg,
              cap ? scale / softcap * 2.f * LOG2E : 0.f, cap ? softcap * LOG2E : 0.f};
#define DS_ROW(K)                                              \
  {                                                            \
    if (dv <= 32) return launch<K, 32, EXT_>(a, nwork, st);    \
    if (dv <= 64) return launch<K, 64, EXT_>(a, nwork, st);    \
    if (dv <= 128) return launch<K, 128, EXT_>(a, nwork, st);  \
    if (dv <= 256) return launch<K, 256, EXT_>(a, nwork, st);  \
  }
  if (dk <= 32) DS_ROW(32)
  else if (dk <= 64) DS_ROW(64)
  else if (dk <= 128) DS_ROW(128)
  else if (dk <= 256) DS_ROW(256)
#undef DS_ROW
  return (int)hipErrorInvalidValue;
}
