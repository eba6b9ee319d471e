// Module of the ops that only models with residual streams use: multi-stream residual + norm, gated delta rule, clamped
// gated activation. A shared object of its own, so that serving a model compiles the mechanisms it has and no others.
#include "bind_util.h"

extern "C" {
int ds_stream_norm(float*, const void*, const int*, const void*, const int*, int, int, const float*, const float*, float,
                   const float*, const float*, void*, int, float, int, hipStream_t);
int ds_clamped_glu(const void*, void*, int64_t, int, float, float, float, int, hipStream_t);
int ds_delta_prepare(const void*, const float*, const void*, const float*, const float*, const int*, const int*,
                     const int*, const int*, float*, void*, float*, int, int, int, int, int, int, int, hipStream_t);
int ds_delta_recur(const float*, const void*, const float*, const void*, const float*, float, float*, void*, const int*,
                   int, const int*, const int*, const int*, void*, int, int, int, int, int, int, int, hipStream_t);
int64_t ds_delta_chunk_ws(int, int, int, int);
int ds_delta_chunk(const float*, const void*, const float*, const void*, const float*, float, float*, void*, const int*,
                   int, const int*, int, const int*, const int*, const int*, float*, float*, void*, int, int, int, int,
                   int, int, int, hipStream_t);
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
  m.def("delta_prepare", &delta_prepare);
  m.def("delta_recur", &delta_recur);
  m.def("delta_chunk", &delta_chunk);
}
