// Module of attention over the paged cache in a ragged batch: QKV epilogues (norms, rotation, cache append), prefill and decode
// with chunked / windowed visibility, score caps and softmax sinks. A shared object of its own, so that serving a model
// compiles the mechanisms it has and no others.
#include "bind_util.h"

extern "C" {
int ds_qk_norm_append(const void*, int64_t, const float*, int, const float*, const float*, float, const void*, int64_t, const float*, const int*,
                      const int*, const int*, int, void*, void*, void*, int, int, int, int, int, int, int, hipStream_t);
int ds_rope_table(const int*, const double*, float*, int, int, float, hipStream_t);
int ds_qk_rope_append(const void*, int64_t, const float*, const float*, const float*, float, const float*, int, float,
                      const int*, const int*, const int*, int, void*, void*, void*, int, int, int, int, int, int, int,
                      hipStream_t);
int ds_paged_generic(const void*, const void*, const void*, void*, const int*, int, const int*, const int*, int, int, int,
                     int, int, int, int, float, float, int, int, const float*, int64_t, const void*, int64_t, int, hipStream_t);
int ds_paged_prefill_ext(const void*, const void*, const void*, void*, const int*, const int*, const int*, const int*, int,
                         int, int, int, int, int, int, int, int, float, float, const float*, const void*, int64_t, int64_t,
                         hipStream_t);
int ds_paged_decode_splits(int, int, int);
int ds_paged_decode_ext(const void*, const void*, const void*, const int*, const int*, float*, float*, void*, int, int,
                        int, int, int, int, int, int, int, float, float, int, int, const float*, const void*, int64_t, int64_t,
                        hipStream_t);
}

namespace {
struct Cache {
  int G, BS, dk, dv;
};
Cache cache_of(const Tensor& kc, const Tensor& vc) {
  need(kc, "k cache"); need(vc, "v cache");
  TORCH_CHECK(kc.dim() == 4 && vc.dim() == 4 && kc.size(0) == vc.size(0) && kc.size(1) == vc.size(1) &&
              kc.size(2) == vc.size(2) && kc.scalar_type() == vc.scalar_type(), "caches [NB, G, BS, dk / dv]");
  return {(int)kc.size(1), (int)kc.size(2), (int)kc.size(3), (int)vc.size(3)};
}

// qkv [T, (H + G) dk + G dv] (rows may be columns of wider ones) -> q [T, H, dk]; k / v into the caches. qw, kw [dk] or none.
// cs [T, half, 2]: turns pairs of neighbours ahead of the norm. vfirst: the same-shaped v columns [T, G dv] (row
// stride free) of an earlier layer, mixed in with weight `lam` [1].
Tensor qk_norm_append(Tensor qkv, OptT qw, OptT kw, double eps, OptT vfirst, OptT lam, Tensor pos, Tensor seq_ids,
                      Tensor block_table, Tensor kc, Tensor vc, int64_t H, OptT cs) {
  need_rows(qkv, "qkv"); need(block_table, "block_table");
  const Cache c = cache_of(kc, vc);
  const int64_t N = (H + c.G) * c.dk + (int64_t)c.G * c.dv, T = qkv.size(0);
  TORCH_CHECK(qkv.size(1) == N, "qk_norm_append: qkv width");
  int64_t half = 0;
  if (has(cs)) {
    half = cs->numel() / 2 / std::max<int64_t>(T, 1);
    TORCH_CHECK(cs->dim() == 3 && cs->size(0) == T && cs->size(2) == 2 && 2 * half <= c.dk, "qk_norm_append: angles [T, half, 2]");
  }
  TORCH_CHECK(qkv.scalar_type() == kc.scalar_type(), "qk_norm_append: projection and cache types differ");
  TORCH_CHECK(block_table.dim() == 2 && block_table.scalar_type() == at::kInt, "block_table [S, M] int32");
  const void* vf = nullptr;
  int64_t vs = 0;
  const float* lp = nullptr;
  if (has(vfirst)) {
    TORCH_CHECK(vfirst->is_cuda() && vfirst->dim() == 2 && vfirst->size(0) == T && vfirst->size(1) == (int64_t)c.G * c.dv &&
                vfirst->stride(1) == 1 && vfirst->scalar_type() == qkv.scalar_type(), "vfirst [T, G dv]");
    vf = vfirst->data_ptr();
    vs = vfirst->stride(0);
    lp = f32(*lam, 1, "lambda");
  }
  auto q = torch::empty({T, H, c.dk}, qkv.options());
  check(ds_qk_norm_append(qkv.data_ptr(), T > 1 ? qkv.stride(0) : N, has(cs) ? f32(*cs, T * half * 2, "angles") : nullptr, (int)half,
                          opt_f32(qw, c.dk, "q norm"), opt_f32(kw, c.dk, "k norm"), (float)eps, vf, vs, lp,
                          i32(pos, T, "pos"), i32(seq_ids, T, "seq_ids"), block_table.data_ptr<int>(),
                          (int)block_table.size(1), q.data_ptr(), kc.data_ptr(), vc.data_ptr(), (int)T, (int)H, c.G, c.dk,
                          c.dv, c.BS, dcode(qkv), stream()), "qk_norm_append");
  return q;
}

// pos [T], freq [half] fp64 -> cos and sin of their products, times mult, [T, half, 2]
Tensor rope_table(Tensor pos, Tensor freq, double mult) {
  const int64_t T = pos.numel(), half = freq.numel();
  auto cs = torch::empty({T, half, 2}, pos.options().dtype(at::kFloat));
  check(ds_rope_table(i32(pos, T, "pos"), f64(freq, "freq"), cs.data_ptr<float>(), (int)T, (int)half, (float)mult, stream()), "rope_table");
  return cs;
}

// qkv [T, >= (H + G) dk + G dv] (rows may be columns of wider ones) -> q [T, H, dk]; k, and v times vmult, into the caches
Tensor qk_rope_append(Tensor qkv, OptT bias, OptT qw, OptT kw, double eps, OptT cs, double vmult, Tensor pos, Tensor seq_ids,
                      Tensor block_table, Tensor kc, Tensor vc, int64_t H) {
  need_rows(qkv, "qkv"); need(block_table, "block_table");
  const Cache c = cache_of(kc, vc);
  const int64_t nqk = (H + c.G) * c.dk, N = nqk + (int64_t)c.G * c.dv, T = qkv.size(0);
  TORCH_CHECK(H > 0 && H % c.G == 0 && qkv.size(1) == N, "qk_rope_append: qkv width");
  TORCH_CHECK(qkv.scalar_type() == kc.scalar_type(), "qk_rope_append: projection and cache types differ");
  TORCH_CHECK(block_table.dim() == 2 && block_table.scalar_type() == at::kInt, "block_table [S, M] int32");
  TORCH_CHECK(nqk * 4 <= 144 * 1024, "qk_rope_append: up to 36864 query and key columns");
  int64_t half = 0;
  if (has(cs)) {
    half = cs->numel() / 2 / std::max<int64_t>(T, 1);
    TORCH_CHECK(cs->dim() == 3 && cs->size(0) == T && cs->size(2) == 2 && 2 * half <= c.dk, "qk_rope_append: angles [T, half, 2]");
  }
  auto q = torch::empty({T, H, c.dk}, qkv.options());
  check(ds_qk_rope_append(qkv.data_ptr(), T > 1 ? qkv.stride(0) : N, opt_f32(bias, N, "bias"), opt_f32(qw, H * c.dk, "q norm"),
                          opt_f32(kw, (int64_t)c.G * c.dk, "k norm"), (float)eps, has(cs) ? f32(*cs, T * half * 2, "angles") : nullptr,
                          (int)half, (float)vmult, i32(pos, T, "pos"), i32(seq_ids, T, "seq_ids"), block_table.data_ptr<int>(),
                          (int)block_table.size(1), q.data_ptr(), kc.data_ptr(), vc.data_ptr(), (int)T, (int)H, c.G, c.dk,
                          c.dv, c.BS, dcode(qkv), stream()), "qk_rope_append");
  return q;
}

// Where attention writes: the given matrix [>= rows, H dv] (its rows may be columns of wider ones), or a new one
struct Out {
  Tensor t;
  int64_t ld;
  Out(const OptT& o, int64_t rows, int64_t H, int64_t dv, const Tensor& q) {
    t = has(o) ? *o : torch::empty({rows, H * dv}, q.options());
    need_rows(t, "out");
    TORCH_CHECK(t.size(0) >= rows && t.size(1) == H * dv && t.scalar_type() == q.scalar_type(), "out [T, H dv]");
    ld = t.size(0) > 1 ? t.stride(0) : H * dv;
  }
};

// Numbers per token and head [rows, H] (columns of a wider matrix), or none
struct Gate {
  const void* p = nullptr;
  int64_t ld = 0;
  Gate(const OptT& g, int64_t rows, int64_t H, const Tensor& q) {
    if (!has(g)) return;
    need_rows(*g, "gate");
    TORCH_CHECK(g->size(0) >= rows && g->size(1) == H && g->scalar_type() == q.scalar_type(), "gate [T, H]");
    p = g->data_ptr();
    ld = g->size(0) > 1 ? g->stride(0) : H;
  }
};

// q [T, H, dk] at positions pos of sequences seq_ids -> o [T, H dv]; exp(sink) of its head joins every denominator, heads come
// out times sigmoid(gate)
Tensor paged_generic(Tensor q, Tensor kc, Tensor vc, Tensor block_table, Tensor pos, Tensor seq_ids, double scale,
                     double softcap, int64_t window, int64_t chunk, OptT sink, OptT out, OptT gate) {
  need(q, "q"); need(block_table, "block_table");
  const Cache c = cache_of(kc, vc);
  const int64_t T = q.size(0), H = q.size(1);
  TORCH_CHECK(q.dim() == 3 && q.size(2) == c.dk && H % c.G == 0 && q.scalar_type() == kc.scalar_type(), "paged_generic: q");
  const Gate g(gate, T, H, q);
  TORCH_CHECK(block_table.dim() == 2 && block_table.scalar_type() == at::kInt, "block_table [S, M] int32");
  TORCH_CHECK(c.dk <= 1024 && c.dv <= 1024, "paged_generic: head sizes up to 1024");
  const Out o(out, T, H, c.dv, q);
  check(ds_paged_generic(q.data_ptr(), kc.data_ptr(), vc.data_ptr(), o.t.data_ptr(), block_table.data_ptr<int>(),
                         (int)block_table.size(1), i32(pos, T, "pos"), i32(seq_ids, T, "seq_ids"), (int)T, (int)H, c.G,
                         c.dk, c.dv, c.dv, c.BS, (float)scale, (float)softcap, (int)window, (int)chunk,
                         opt_f32(sink, H, "sink"), o.ld, g.p, g.ld, dcode(q), stream()), "paged_generic");
  return o.t;
}

bool paged_tiled_ok(int64_t dk, int64_t dv) { return dk % 8 == 0 && dv % 8 == 0 && dk <= 256 && dv <= 256; }

// Prompts and portions: q [T, H, dk] bf16 of every new token; work [n, 2] names (sequence, 128-row block) -> o [T, H dv]
// (rows of sequences the list leaves out are not written).
Tensor paged_prefill(Tensor q, Tensor kc, Tensor vc, Tensor block_table, Tensor start, Tensor cu_q, Tensor work,
                     double scale, double softcap, int64_t window, int64_t chunk, OptT sink, OptT out, OptT gate) {
  need(q, "q"); need(block_table, "block_table");
  const Cache c = cache_of(kc, vc);
  const int64_t T = q.size(0), H = q.size(1), S = start.numel();
  TORCH_CHECK(q.dim() == 3 && q.size(2) == c.dk && H % c.G == 0 && q.scalar_type() == at::kBFloat16 &&
              kc.scalar_type() == at::kBFloat16 && paged_tiled_ok(c.dk, c.dv), "paged_prefill: q / caches");
  TORCH_CHECK(block_table.dim() == 2 && block_table.size(0) == S && block_table.scalar_type() == at::kInt, "block_table");
  TORCH_CHECK(work.dim() == 2 && work.size(1) == 2 && scale > 0, "paged_prefill: work [n, 2], scale > 0");
  const Out o(out, T, H, c.dv, q);
  const Gate g(gate, T, H, q);
  check(ds_paged_prefill_ext(q.data_ptr(), kc.data_ptr(), vc.data_ptr(), o.t.data_ptr(), block_table.data_ptr<int>(),
                             i32(start, S, "start"), i32(cu_q, S + 1, "cu_q"), i32(work, work.numel(), "work"),
                             (int)work.size(0), (int)H, c.G, c.dk, c.dv, c.BS, (int)block_table.size(1), (int)window,
                             (int)chunk, (float)scale, (float)softcap, opt_f32(sink, H, "sink"), g.p, g.ld, o.ld, stream()),
        "paged_prefill");
  return o.t;
}

// One new token per sequence: q [B, H, dk] bf16, the first B rows of the tables -> out[:B] of [.., H dv]
void paged_decode(Tensor q, Tensor kc, Tensor vc, Tensor block_table, Tensor seq_lens, int64_t max_len, double scale,
                  double softcap, int64_t window, int64_t chunk, Tensor out, OptT sink, OptT gate) {
  need(q, "q"); need(block_table, "block_table");
  const Cache c = cache_of(kc, vc);
  const int64_t B = q.size(0), H = q.size(1);
  TORCH_CHECK(q.dim() == 3 && q.size(2) == c.dk && H % c.G == 0 && q.scalar_type() == at::kBFloat16 &&
              kc.scalar_type() == at::kBFloat16 && paged_tiled_ok(c.dk, c.dv), "paged_decode: q / caches");
  TORCH_CHECK(block_table.dim() == 2 && block_table.size(0) >= B && block_table.scalar_type() == at::kInt &&
              block_table.size(1) * c.BS >= max_len, "block_table");
  const Out o(out, B, H, c.dv, q);
  const Gate g(gate, B, H, q);
  int64_t span = max_len;
  if (window > 0) span = std::min(span, window);
  if (chunk > 0) span = std::min(span, chunk);
  const int splits = ds_paged_decode_splits((int)B, c.G, (int)span);
  Tensor acc, ml;
  if (splits > 1) {
    auto fo = q.options().dtype(at::kFloat);
    acc = torch::empty({B, H, splits, c.dv}, fo);
    ml = torch::empty({B, H, splits, 2}, fo);
  }
  check(ds_paged_decode_ext(q.data_ptr(), kc.data_ptr(), vc.data_ptr(), block_table.data_ptr<int>(),
                            i32(seq_lens, seq_lens.numel(), "seq_lens"), splits > 1 ? acc.data_ptr<float>() : nullptr,
                            splits > 1 ? ml.data_ptr<float>() : nullptr, o.t.data_ptr(), (int)B, (int)H, c.G, c.dk, c.dv,
                            c.BS, (int)block_table.size(1), (int)span, splits, (float)scale, (float)softcap, (int)window,
                            (int)chunk, opt_f32(sink, H, "sink"), g.p, g.ld, o.ld, stream()), "paged_decode");
}
}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("qk_norm_append", &qk_norm_append);
  m.def("rope_table", &rope_table);
  m.def("qk_rope_append", &qk_rope_append);
  m.def("paged_generic", &paged_generic);
  m.def("paged_tiled_ok", &paged_tiled_ok);
  m.def("paged_prefill", &paged_prefill);
  m.def("paged_decode", &paged_decode);
}
