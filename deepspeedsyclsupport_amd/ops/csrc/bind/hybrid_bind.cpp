// Module of the hybrid decoder's ops: multi-stream residual + norm, QKV epilogue with per-head norms, ragged paged
// attention with chunked / windowed visibility and score capping, gated delta rule, clamped gated activation. A shared
// object of its own, so that serving such a model compiles only this and the decode products (gemv_bind.cpp).
#include "bind_util.h"

extern "C" {
int ds_stream_norm(float*, const void*, const int*, const void*, const int*, int, int, const float*, const float*, float,
                   const float*, const float*, void*, int, float, int, hipStream_t);
int ds_clamped_glu(const void*, void*, int64_t, int, float, float, float, int, hipStream_t);
int ds_qk_norm_append(const void*, const float*, const float*, float, const void*, int64_t, const float*, const int*,
                      const int*, const int*, int, void*, void*, void*, int, int, int, int, int, int, int, hipStream_t);
int ds_paged_generic(const void*, const void*, const void*, void*, const int*, int, const int*, const int*, int, int, int,
                     int, int, int, int, float, float, int, int, const float*, int, hipStream_t);
int ds_delta_prepare(const void*, const float*, const void*, const float*, const float*, const int*, const int*,
                     const int*, const int*, float*, void*, float*, int, int, int, int, int, int, int, hipStream_t);
int ds_delta_recur(const float*, const void*, const float*, const void*, const float*, float, float*, void*, const int*,
                   int, const int*, const int*, const int*, void*, int, int, int, int, int, int, int, hipStream_t);
int64_t ds_delta_chunk_ws(int, int, int, int);
int ds_delta_chunk(const float*, const void*, const float*, const void*, const float*, float, float*, void*, const int*,
                   int, const int*, int, const int*, const int*, const int*, float*, float*, void*, int, int, int, int,
                   int, int, int, hipStream_t);
int ds_paged_prefill_ext(const void*, const void*, const void*, void*, const int*, const int*, const int*, const int*, int,
                         int, int, int, int, int, int, int, int, float, float, hipStream_t);
int ds_paged_decode_splits(int, int, int);
int ds_paged_decode_ext(const void*, const void*, const void*, const int*, const int*, float*, float*, void*, int, int,
                        int, int, int, int, int, int, int, float, float, int, int, hipStream_t);
}

namespace {
// x [T, S, W] fp32 (updated in place unless `rows`). Either y [T, W] with mix [S, S] / out [S] (finish a sublayer), or
// ids [T] + embed [V, W] (start of the model). Returns the normed rows [R, W] in y's / embed's type.
Tensor stream_norm(Tensor x, OptT y, OptT mix, OptT out, double m, OptT in, Tensor w, double eps, OptT ids, OptT embed,
                   OptT rows) {
  need(x, "x");
  TORCH_CHECK(x.scalar_type() == at::kFloat && x.dim() == 3, "stream_norm: x [T, S, W] fp32");
  const int64_t T = x.size(0), S = x.size(1), W = x.size(2);
  TORCH_CHECK(S >= 1 && S <= 8, "stream_norm: 1 to 8 streams");
  TORCH_CHECK(W <= 15360, "stream_norm: width up to 15360");
  TORCH_CHECK(has(y) != has(embed), "stream_norm: y or embed");
  const Tensor& src = has(y) ? *y : *embed;
  need(src, "y / embed");
  TORCH_CHECK(src.size(-1) == W, "stream_norm: width");
  const float *mp = nullptr, *op = nullptr;
  const int *ip = nullptr, *rp = nullptr;
  if (has(y)) {
    TORCH_CHECK(y->numel() == T * W, "stream_norm: y [T, W]");
    mp = f32(*mix, S * S, "mix");
    op = f32(*out, S, "out");
  } else {
    ip = i32(*ids, T, "ids");
    TORCH_CHECK(!has(rows), "stream_norm: no row list at the start");
  }
  int64_t R = T;
  if (has(rows)) {
    R = rows->numel();
    rp = i32(*rows, R, "rows");
  }
  auto normed = torch::empty({R, W}, src.options());
  check(ds_stream_norm(x.data_ptr<float>(), has(y) ? y->data_ptr() : nullptr, ip, has(embed) ? embed->data_ptr() : nullptr,
                       rp, (int)R, (int)S, mp, op, (float)m, has(in) ? f32(*in, S, "in") : nullptr,
                       f32(w, W, "norm weight"), normed.data_ptr(), (int)W, (float)eps, dcode(src), stream()),
        "stream_norm");
  return normed;
}

Tensor clamped_glu(Tensor gu, double limit, double alpha, double shift) {
  need(gu, "gate_up");
  const int64_t F = gu.size(-1) / 2, rows = gu.numel() / gu.size(-1);
  TORCH_CHECK(gu.size(-1) % 2 == 0, "clamped_glu: [.., 2F]");
  auto sizes = gu.sizes().vec();
  sizes.back() = F;
  auto out = torch::empty(sizes, gu.options());
  check(ds_clamped_glu(gu.data_ptr(), out.data_ptr(), rows, (int)F, (float)limit, (float)alpha, (float)shift, dcode(gu),
                       stream()), "clamped_glu");
  return out;
}

struct Cache {
  int G, BS, dk, dv;
};
Cache cache_of(const Tensor& kc, const Tensor& vc) {
  need(kc, "k cache"); need(vc, "v cache");
  TORCH_CHECK(kc.dim() == 4 && vc.dim() == 4 && kc.size(0) == vc.size(0) && kc.size(1) == vc.size(1) &&
              kc.size(2) == vc.size(2) && kc.scalar_type() == vc.scalar_type(), "caches [NB, G, BS, dk / dv]");
  return {(int)kc.size(1), (int)kc.size(2), (int)kc.size(3), (int)vc.size(3)};
}

// qkv [T, (H + G) dk + G dv] -> q [T, H, dk]; k / v into the caches. vfirst: the same-shaped v columns [T, G dv] (row
// stride free) of an earlier layer, mixed in with weight `lam` [1].
Tensor qk_norm_append(Tensor qkv, Tensor qw, Tensor kw, double eps, OptT vfirst, OptT lam, Tensor pos, Tensor seq_ids,
                      Tensor block_table, Tensor kc, Tensor vc, int64_t H) {
  need(qkv, "qkv"); need(block_table, "block_table");
  const Cache c = cache_of(kc, vc);
  const int64_t N = (H + c.G) * c.dk + (int64_t)c.G * c.dv, T = qkv.numel() / N;
  TORCH_CHECK(qkv.numel() == T * N && qkv.size(-1) == N, "qk_norm_append: qkv width");
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
  check(ds_qk_norm_append(qkv.data_ptr(), f32(qw, c.dk, "q norm"), f32(kw, c.dk, "k norm"), (float)eps, vf, vs, lp,
                          i32(pos, T, "pos"), i32(seq_ids, T, "seq_ids"), block_table.data_ptr<int>(),
                          (int)block_table.size(1), q.data_ptr(), kc.data_ptr(), vc.data_ptr(), (int)T, (int)H, c.G, c.dk,
                          c.dv, c.BS, dcode(qkv), stream()), "qk_norm_append");
  return q;
}

// q [T, H, dk] at positions pos of sequences seq_ids -> o [T, H, dv]
Tensor paged_generic(Tensor q, Tensor kc, Tensor vc, Tensor block_table, Tensor pos, Tensor seq_ids, double scale,
                     double softcap, int64_t window, int64_t chunk) {
  need(q, "q"); need(block_table, "block_table");
  const Cache c = cache_of(kc, vc);
  const int64_t T = q.size(0), H = q.size(1);
  TORCH_CHECK(q.dim() == 3 && q.size(2) == c.dk && H % c.G == 0 && q.scalar_type() == kc.scalar_type(), "paged_generic: q");
  TORCH_CHECK(block_table.dim() == 2 && block_table.scalar_type() == at::kInt, "block_table [S, M] int32");
  TORCH_CHECK(c.dk <= 1024 && c.dv <= 1024, "paged_generic: head sizes up to 1024");
  auto o = torch::empty({T, H, c.dv}, q.options());
  check(ds_paged_generic(q.data_ptr(), kc.data_ptr(), vc.data_ptr(), o.data_ptr(), block_table.data_ptr<int>(),
                         (int)block_table.size(1), i32(pos, T, "pos"), i32(seq_ids, T, "seq_ids"), (int)T, (int)H, c.G,
                         c.dk, c.dv, c.dv, c.BS, (float)scale, (float)softcap, (int)window, (int)chunk, nullptr, dcode(q),
                         stream()), "paged_generic");
  return o;
}

bool paged_tiled_ok(int64_t dk, int64_t dv) { return dk % 8 == 0 && dv % 8 == 0 && dk <= 256 && dv <= 256; }

// Prompts and portions: q [T, H, dk] bf16 of every new token; work [n, 2] names (sequence, 128-row block) -> o [T, H, dv]
// (rows of sequences the list leaves out are not written).
Tensor paged_prefill(Tensor q, Tensor kc, Tensor vc, Tensor block_table, Tensor start, Tensor cu_q, Tensor work,
                     double scale, double softcap, int64_t window, int64_t chunk) {
  need(q, "q"); need(block_table, "block_table");
  const Cache c = cache_of(kc, vc);
  const int64_t T = q.size(0), H = q.size(1), S = start.numel();
  TORCH_CHECK(q.dim() == 3 && q.size(2) == c.dk && H % c.G == 0 && q.scalar_type() == at::kBFloat16 &&
              kc.scalar_type() == at::kBFloat16 && paged_tiled_ok(c.dk, c.dv), "paged_prefill: q / caches");
  TORCH_CHECK(block_table.dim() == 2 && block_table.size(0) == S && block_table.scalar_type() == at::kInt, "block_table");
  TORCH_CHECK(work.dim() == 2 && work.size(1) == 2 && scale > 0, "paged_prefill: work [n, 2], scale > 0");
  auto o = torch::empty({T, H, c.dv}, q.options());
  check(ds_paged_prefill_ext(q.data_ptr(), kc.data_ptr(), vc.data_ptr(), o.data_ptr(), block_table.data_ptr<int>(),
                             i32(start, S, "start"), i32(cu_q, S + 1, "cu_q"), i32(work, work.numel(), "work"),
                             (int)work.size(0), (int)H, c.G, c.dk, c.dv, c.BS, (int)block_table.size(1), (int)window,
                             (int)chunk, (float)scale, (float)softcap, stream()), "paged_prefill");
  return o;
}

// One new token per sequence: q [B, H, dk] bf16, the first B rows of the tables -> out[:B] of [.., H, dv]
void paged_decode(Tensor q, Tensor kc, Tensor vc, Tensor block_table, Tensor seq_lens, int64_t max_len, double scale,
                  double softcap, int64_t window, int64_t chunk, Tensor out) {
  need(q, "q"); need(block_table, "block_table"); need(out, "out");
  const Cache c = cache_of(kc, vc);
  const int64_t B = q.size(0), H = q.size(1);
  TORCH_CHECK(q.dim() == 3 && q.size(2) == c.dk && H % c.G == 0 && q.scalar_type() == at::kBFloat16 &&
              kc.scalar_type() == at::kBFloat16 && paged_tiled_ok(c.dk, c.dv), "paged_decode: q / caches");
  TORCH_CHECK(block_table.dim() == 2 && block_table.size(0) >= B && block_table.scalar_type() == at::kInt &&
              block_table.size(1) * c.BS >= max_len, "block_table");
  TORCH_CHECK(out.dim() == 3 && out.size(0) >= B && out.size(1) == H && out.size(2) == c.dv &&
              out.scalar_type() == at::kBFloat16, "paged_decode: out");
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
                            splits > 1 ? ml.data_ptr<float>() : nullptr, out.data_ptr(), (int)B, (int)H, c.G, c.dk, c.dv,
                            c.BS, (int)block_table.size(1), (int)span, splits, (float)scale, (float)softcap, (int)window,
                            (int)chunk, stream()), "paged_decode");
}

void delta_dims_ok(int64_t Hk, int64_t H, int64_t dk, int64_t dv, int64_t taps) {
  TORCH_CHECK(Hk > 0 && H % Hk == 0 && dk > 0 && dv > 0 && taps >= 1, "delta rule: head counts / sizes");
  TORCH_CHECK(dk <= 256 && dv <= 256, "delta rule: head sizes up to 256");
}

// proj [T, 2 Hk dk + 2 H dv + 2 H] -> (qk fp32 [2, Hk, T, dk padded to 4], v [H, T, dv], gb fp32 [T, 2, H]: log decay, beta)
std::vector<Tensor> delta_prepare(Tensor proj, Tensor conv_w, Tensor conv_state, Tensor a_log, Tensor dt_bias,
                                  Tensor seq_ids, Tensor cu, Tensor start, Tensor slots, int64_t Hk, int64_t H, int64_t dk,
                                  int64_t dv) {
  need(proj, "proj"); need(conv_state, "conv_state");
  const int64_t C = 2 * Hk * dk + H * dv, NP = C + H * dv + 2 * H, T = proj.numel() / NP, taps = conv_w.size(-1);
  delta_dims_ok(Hk, H, dk, dv, taps);
  TORCH_CHECK(proj.size(-1) == NP, "delta_prepare: projection width");
  TORCH_CHECK(conv_state.dim() == 3 && conv_state.size(1) == taps - 1 && conv_state.size(2) == C &&
              conv_state.scalar_type() == proj.scalar_type(), "delta_prepare: conv_state [slots, taps-1, C]");
  const int64_t S = start.numel();
  auto fo = proj.options().dtype(at::kFloat);
  auto qk = torch::empty({2, Hk, T, (dk + 3) / 4 * 4}, fo);  // zero padded rows
  auto v = torch::empty({H, T, dv}, proj.options());
  auto gb = torch::empty({T, 2, H}, fo);
  check(ds_delta_prepare(proj.data_ptr(), f32(conv_w, C * taps, "conv_w"), conv_state.data_ptr(), f32(a_log, H, "A_log"),
                         f32(dt_bias, H, "dt_bias"), i32(seq_ids, T, "seq_ids"), i32(cu, S + 1, "cu"),
                         i32(start, S, "start"), i32(slots, S, "slots"), qk.data_ptr<float>(), v.data_ptr(),
                         gb.data_ptr<float>(), (int)T, (int)Hk, (int)H, (int)dk, (int)dv, (int)taps, dcode(proj), stream()),
        "delta_prepare");
  return {qk, v, gb};
}

// Runs the sequences in `list`; writes their rows of out [T, H dv] and their state slots.
void delta_recur(Tensor qk, Tensor v, Tensor gb, Tensor proj, Tensor norm_w, double eps, Tensor state, Tensor conv_state,
                 Tensor list, Tensor cu, Tensor start, Tensor slots, Tensor out, int64_t dk) {
  need(proj, "proj"); need(v, "v"); need(state, "state"); need(conv_state, "conv_state"); need(out, "out");
  const int64_t T = v.size(1), H = v.size(0), dv = v.size(2), Hk = qk.size(1), S = start.numel();
  const int64_t taps = conv_state.size(1) + 1;
  delta_dims_ok(Hk, H, dk, dv, taps);
  TORCH_CHECK(state.scalar_type() == at::kFloat && state.dim() == 4 && state.size(1) == H && state.size(2) == dv &&
              state.size(3) == (dk + 3) / 4 * 4 && state.size(0) == conv_state.size(0), "delta: state [slots, H, dv, dk padded to 4] fp32");
  TORCH_CHECK(conv_state.size(2) == 2 * Hk * dk + H * dv, "delta: conv_state");
  TORCH_CHECK(proj.numel() == T * (2 * Hk * dk + 2 * H * dv + 2 * H) && out.numel() == T * H * dv, "delta: proj / out");
  TORCH_CHECK(v.scalar_type() == proj.scalar_type() && out.scalar_type() == proj.scalar_type() &&
              conv_state.scalar_type() == proj.scalar_type(), "delta: types");
  check(ds_delta_recur(f32(qk, T * 2 * Hk * ((dk + 3) / 4 * 4), "qk"), v.data_ptr(), f32(gb, T * 2 * H, "gb"), proj.data_ptr(),
                       f32(norm_w, dv, "norm"), (float)eps, state.data_ptr<float>(), conv_state.data_ptr(),
                       i32(list, list.numel(), "list"), (int)list.numel(), i32(cu, S + 1, "cu"), i32(start, S, "start"),
                       i32(slots, S, "slots"), out.data_ptr(), (int)T, (int)Hk, (int)H, (int)dk, (int)dv, (int)taps,
                       dcode(proj), stream()), "delta_recur");
}

// The same for long portions, by chunks of 64 tokens: seqs [n, 2] (sequence, its first entry in work), work [m, 2]
// (sequence, chunk).
void delta_chunk(Tensor qk, Tensor v, Tensor gb, Tensor proj, Tensor norm_w, double eps, Tensor state, Tensor conv_state,
                 Tensor seqs, Tensor work, Tensor cu, Tensor start, Tensor slots, Tensor out, int64_t dk) {
  need(proj, "proj"); need(v, "v"); need(state, "state"); need(conv_state, "conv_state"); need(out, "out");
  const int64_t T = v.size(1), H = v.size(0), dv = v.size(2), Hk = qk.size(1), S = start.numel();
  const int64_t taps = conv_state.size(1) + 1;
  delta_dims_ok(Hk, H, dk, dv, taps);
  TORCH_CHECK(state.scalar_type() == at::kFloat && state.dim() == 4 && state.size(1) == H && state.size(2) == dv &&
              state.size(3) == (dk + 3) / 4 * 4 && state.size(0) == conv_state.size(0), "delta: state [slots, H, dv, dk padded to 4] fp32");
  TORCH_CHECK(conv_state.size(2) == 2 * Hk * dk + H * dv, "delta: conv_state");
  TORCH_CHECK(proj.numel() == T * (2 * Hk * dk + 2 * H * dv + 2 * H) && out.numel() == T * H * dv, "delta: proj / out");
  TORCH_CHECK(v.scalar_type() == proj.scalar_type() && out.scalar_type() == proj.scalar_type() &&
              conv_state.scalar_type() == proj.scalar_type(), "delta: types");
  TORCH_CHECK(seqs.dim() == 2 && seqs.size(1) == 2 && work.dim() == 2 && work.size(1) == 2, "delta_chunk: lists");
  const int64_t nw = work.size(0);
  auto fo = proj.options().dtype(at::kFloat);
  auto ws = torch::empty({ds_delta_chunk_ws((int)nw, (int)H, (int)dk, (int)dv)}, fo);
  auto o = torch::empty({H, T, dv}, fo);
  check(ds_delta_chunk(f32(qk, T * 2 * Hk * ((dk + 3) / 4 * 4), "qk"), v.data_ptr(), f32(gb, T * 2 * H, "gb"), proj.data_ptr(),
                       f32(norm_w, dv, "norm"), (float)eps, state.data_ptr<float>(), conv_state.data_ptr(),
                       i32(seqs, seqs.numel(), "seqs"), (int)seqs.size(0), i32(work, work.numel(), "work"), (int)nw,
                       i32(cu, S + 1, "cu"), i32(start, S, "start"), i32(slots, S, "slots"), ws.data_ptr<float>(),
                       o.data_ptr<float>(), out.data_ptr(), (int)T, (int)Hk, (int)H, (int)dk, (int)dv, (int)taps, dcode(proj),
                       stream()), "delta_chunk");
}
}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("stream_norm", &stream_norm, py::arg("x"), py::arg("y"), py::arg("mix"), py::arg("out"), py::arg("m"),
        py::arg("in_"), py::arg("w"), py::arg("eps"), py::arg("ids") = py::none(), py::arg("embed") = py::none(),
        py::arg("rows") = py::none());
  m.def("clamped_glu", &clamped_glu);
  m.def("qk_norm_append", &qk_norm_append);
  m.def("paged_generic", &paged_generic);
  m.def("delta_prepare", &delta_prepare);
  m.def("delta_recur", &delta_recur);
  m.def("delta_chunk", &delta_chunk);
  m.def("paged_tiled_ok", &paged_tiled_ok);
  m.def("paged_prefill", &paged_prefill);
  m.def("paged_decode", &paged_decode);
}
