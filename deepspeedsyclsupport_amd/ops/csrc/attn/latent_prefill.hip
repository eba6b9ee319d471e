// Attention of prompts and long portions over keys and values expanded from cached latents (see latent_ops.hip), CDNA4
// (gfx950): entry point. The kernel is paged_prefill_core.h's.
#include "paged_prefill_core.h"

// q / o [T, H, dn + r] (ldq elements from token to token) / [T, H, dv] bf16, rotated; kv [rows, H (dn + dv)]: expanded context rows, keys of all heads, then
// values; ctx [rows, ldr]: the latents' rows, whose columns rot0 .. rot0 + r are the rotated key part. kv_offs: place of the
// contexts of sequences first, first + 1, ..., kv_first: their first keys (multiples of 64, none behind what the window lets the
// first new token see; null: 0); work [nwork, 2] (sequence, 128-row query block). Tiles of 64 keys are
// read whole: 64 (finite) rows must exist behind the last context in kv and ctx.
extern "C" int ds_latent_prefill(const void* q, const void* kv, const void* ctx, void* o, const int* start, const int* cu_q,
                                 const int* work, int nwork, const int* kv_offs, const int* kv_first, int first, int64_t ldq,
                                 int window, int H, int dn, int r, int dv,
                                 int ldr, int rot0, const float* sink, float scale, hipStream_t st) {
  if (nwork <= 0) return 0;
  const int dk = dn + r;
  if (ldq % 8 || ((uintptr_t)q & 15) || ldq < (int64_t)H * dk || window < 0 || H <= 0 || scale <= 0.f || dn <= 0 || r < 0 || dv <= 0 || dn % 8 || r % 8 || dv % 8 || ldr % 8 || rot0 % 8 ||
      (int64_t)nwork * H > INT32_MAX)
    return (int)hipErrorInvalidValue;
  PagedArgs a{};
  a.q = (const bf16*)q;
  a.kc = (const bf16*)kv;
  a.vc = (const bf16*)ctx;
  a.o = (bf16*)o;
  a.start = start;
  a.cu_q = cu_q;
  a.work = work;
  a.Hq = a.Hk = H;
  a.c = scale * 1.4426950408889634f;
  a.inv_scale = 1.f / scale;
  a.dk = dk;
  a.dv = dv;
  a.sink = sink;
  a.kv_offs = kv_offs;
  a.kv_first = kv_first;
  a.first = first;
  a.ldq = ldq;
  a.window = window;
  a.dn = dn;
  a.ldk = H * (dn + dv);
  a.ldr = ldr;
  a.rot0 = rot0;
  a.ldo = (int64_t)H * dv;
#define DS_ROW(K)                                               \
  {                                                             \
    if (dv <= 32) return launch<K, 32, LATENT>(a, nwork, st);   \
    if (dv <= 64) return launch<K, 64, LATENT>(a, nwork, st);   \
    if (dv <= 128) return launch<K, 128, LATENT>(a, nwork, st); \
    if (dv <= 256) return launch<K, 256, LATENT>(a, nwork, st); \
  }
  if (dk <= 32) DS_ROW(32)
  else if (dk <= 64) DS_ROW(64)
  else if (dk <= 128) DS_ROW(128)
  else if (dk <= 192) DS_ROW(192)
  else if (dk <= 256) DS_ROW(256)
#undef DS_ROW
  return (int)hipErrorInvalidValue;
}

extern "C" int ds_latent_prefill_ok(int dn, int r, int dv) {
  return dn > 0 && r >= 0 && dv > 0 && dn % 8 == 0 && r % 8 == 0 && dv % 8 == 0 && dn + r <= 256 && dv <= 256;
}
