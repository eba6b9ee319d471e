// Module of the ops of post-norm hybrid decoders: norms on sublayer outputs, token-side gates, latent attention. A shared
// object of its own, so that serving a model compiles the mechanisms it has and no others.
#include "bind_util.h"

extern "C" {
int ds_post_norm(float*, const void*, const float*, const int*, const void*, const int*, int, const float*, float, void*, int,
                 float, int, hipStream_t);
int ds_gelu(const void*, void*, int64_t, int, hipStream_t);
int ds_token_gate(const void*, const int*, const void*, int64_t, void*, int64_t, int, int, hipStream_t);
int ds_latent_prepare(const void*, int64_t, const float*, const float*, float, const double*, float, int, const int*, const int*, const int*,
                      int, void*, void*, int, int, int, int, int, int, hipStream_t);
int ds_rotate_tail(void*, int64_t, int, int, int, int, const double*, float, int, const int*, int, hipStream_t);
int ds_head_linear(const void*, const void*, void*, int, int, int, int, int, int, int, int64_t, int, const double*, float,
                   const int*, int, hipStream_t);
int ds_latent_gather(const void*, const int*, int, const int*, const int*, int, int, void*, int64_t, int, int, int, hipStream_t);
int ds_paged_generic(const void*, const void*, const void*, void*, const int*, int, const int*, const int*, int, int, int,
                     int, int, int, int, float, float, int, int, const float*, int64_t, const void*, int64_t, int, hipStream_t);
int ds_latent_decode_ok(int, int);
void ds_latent_decode_plan(int, int, int, int, int, int*, int*);
int ds_latent_decode(const void*, const void*, void*, float*, float*, const int*, int, const int*, const int*, int, int, int,
                     int, int, int, int, int, int, int, int, int, const float*, float, hipStream_t);
int ds_latent_prefill_ok(int, int, int);
int ds_latent_prefill(const void*, const void*, const void*, void*, const int*, const int*, const int*, int, const int*,
                      const int*, int, int64_t, int, int, int, int, int, int, int, const float*, float, hipStream_t);
}

namespace {
void table(const Tensor& bt, int64_t seqs) {
  need(bt, "block_table");
  TORCH_CHECK(bt.dim() == 2 && bt.scalar_type() == at::kInt && bt.size(0) >= seqs, "block_table [S, M] int32");
}

// x [T, W] fp32, in place. y [T, W] + w: x += y / rms(y) w; ids + embed: x = embed[ids]. -> x in y's / embed's type; with
// rows: those rows of the sum, normed by final_w, times mult (x stays)
Tensor post_norm(Tensor x, OptT y, OptT w, double eps, OptT ids, OptT embed, OptT rows, OptT final_w, double mult) {
  need(x, "x");
  TORCH_CHECK(x.scalar_type() == at::kFloat && x.dim() == 2, "post_norm: x [T, W] fp32");
  const int64_t T = x.size(0), W = x.size(1);
  TORCH_CHECK(has(y) != has(embed), "post_norm: y or embed");
  const Tensor& src = has(y) ? *y : *embed;
  need(src, "y / embed");
  TORCH_CHECK(src.size(-1) == W && (has(embed) || src.numel() == T * W), "post_norm: width");
  TORCH_CHECK(!has(rows) || has(y), "post_norm: no row list at the start");
  const int64_t R = has(rows) ? rows->numel() : T;
  auto out = torch::empty({R, W}, src.options());
  check(ds_post_norm(x.data_ptr<float>(), has(y) ? y->data_ptr() : nullptr, has(y) ? f32(*w, W, "norm weight") : nullptr,
                     has(embed) ? i32(*ids, T, "ids") : nullptr, has(embed) ? embed->data_ptr() : nullptr,
                     has(rows) ? i32(*rows, R, "rows") : nullptr, (int)R, has(rows) ? f32(*final_w, W, "final norm") : nullptr,
                     (float)mult, out.data_ptr(), (int)W, (float)eps, dcode(src), stream()), "post_norm");
  return out;
}

Tensor gelu(Tensor x) {
  need(x, "x");
  auto out = torch::empty_like(x);
  check(ds_gelu(x.data_ptr(), out.data_ptr(), x.numel(), dcode(x), stream()), "gelu");
  return out;
}

Tensor token_gate(Tensor g, Tensor ids, Tensor table_, int64_t first) {
  need(g, "g"); need(table_, "table");
  const int64_t D = g.size(-1), T = g.numel() / D;
  TORCH_CHECK(table_.dim() == 2 && table_.scalar_type() == g.scalar_type() && first >= 0 && first + D <= table_.size(1),
              "token_gate: table");
  auto out = torch::empty_like(g);
  check(ds_token_gate(g.data_ptr(), i32(ids, T, "ids"), (const char*)table_.data_ptr() + first * table_.element_size(),
                      table_.size(1), out.data_ptr(), T, (int)D, dcode(g), stream()), "token_gate");
  return out;
}

// ---------------------------------------------------------------------------------------------- latent attention
struct Lat {
  int BS, W;
};
Lat lat_of(const Tensor& lat) {
  need(lat, "latents");
  TORCH_CHECK(lat.dim() == 4 && lat.size(1) == 1, "latents [blocks, 1, block, width]");
  return {(int)lat.size(2), (int)lat.size(3)};
}

// down [T, Q + R + r] (rows may be columns of wider ones) -> normed query latent [T, Q] (Q 0: none); the cached rows [R + r] of
// every token are written. mult: factor of cosine and sine
OptT latent_prepare(Tensor down, OptT qw, Tensor kvw, double eps, Tensor freq, double mult, Tensor pos, Tensor seq_ids, Tensor bt,
                    Tensor lat, int64_t Q) {
  need_rows(down, "down"); table(bt, 1);
  const Lat c = lat_of(lat);
  const int64_t R = kvw.numel(), r = c.W - R, T = down.size(0), half = freq.numel();
  TORCH_CHECK(down.size(1) >= Q + c.W && r >= 0 && 2 * half <= r && down.scalar_type() == lat.scalar_type(),
              "latent_prepare: widths / types");
  OptT cq;
  if (Q) cq = torch::empty({T, Q}, down.options());
  check(ds_latent_prepare(down.data_ptr(), T > 1 ? down.stride(0) : down.size(1), Q ? f32(*qw, Q, "q norm") : nullptr,
                          f32(kvw, R, "kv norm"), (float)eps, f64(freq, "freq"), (float)mult, (int)half, i32(pos, T, "pos"),
                          i32(seq_ids, T, "seq_ids"), bt.data_ptr<int>(), (int)bt.size(1), lat.data_ptr(),
                          Q ? cq->data_ptr() : nullptr, (int)T, (int)Q, (int)R, (int)r, c.BS, dcode(down), stream()),
        "latent_prepare");
  return cq;
}

// q [T, H, row] whose tokens may lie further apart than their heads need; elements from token to token
int64_t need_heads(const Tensor& q, const char* name) {
  TORCH_CHECK(q.is_cuda() && q.dim() == 3 && q.stride(2) == 1 && (q.size(1) <= 1 || q.stride(1) == q.size(2)) &&
              (q.size(0) <= 1 || q.stride(0) >= q.size(1) * q.size(2)), name, ": [T, H, row], heads side by side");
  return q.size(0) > 1 ? q.stride(0) : q.size(1) * q.size(2);
}

// Last columns of every head of q [T, H, row] (the ones behind row - r), rotated in place. q may be rows of a larger batch.
void rotate_tail(Tensor q, Tensor freq, Tensor pos, int64_t r, double mult) {
  const int64_t ld = need_heads(q, "q");
  TORCH_CHECK(r <= q.size(2) && 2 * freq.numel() <= r, "rotate_tail: q [T, H, row]");
  check(ds_rotate_tail(q.data_ptr(), ld, (int)q.size(0), (int)q.size(1), (int)q.size(2), (int)r, f64(freq, "freq"), (float)mult,
                       (int)freq.numel(), i32(pos, q.size(0), "pos"), dcode(q), stream()), "rotate_tail");
}

// y[t, h] = w[h] x[t, h, :K]: x [T, H, xrow], w [H, N, K]. With freq and pos the columns of x behind K are rotated and put
// behind the N of y. `out`: [T, H, N] to write into.
Tensor head_linear(Tensor x, Tensor w, OptT freq, OptT pos, OptT out, double mult) {
  const int64_t ldx = need_heads(x, "x");
  need(w, "w");
  TORCH_CHECK(w.dim() == 3 && w.size(0) == x.size(1) && w.size(2) <= x.size(2) &&
              x.scalar_type() == w.scalar_type(), "head_linear: x [T, H, >= K], w [H, N, K]");
  const int64_t T = x.size(0), H = x.size(1), N = w.size(1), K = w.size(2), r = has(freq) ? x.size(2) - K : 0;
  const int64_t half = has(freq) ? freq->numel() : 0;
  TORCH_CHECK(2 * half <= r || !has(freq), "head_linear: rotated columns");
  Tensor y = has(out) ? *out : torch::empty({T, H, N + r}, x.options());
  need(y, "out");
  TORCH_CHECK(y.dim() == 3 && y.size(0) == T && y.size(1) == H && y.size(2) == N + r && y.scalar_type() == x.scalar_type(),
              "head_linear: out");
  check(ds_head_linear(x.data_ptr(), w.data_ptr(), y.data_ptr(), (int)T, (int)H, (int)N, (int)K, (int)x.size(2), (int)y.size(2),
                       (int)r, ldx, (int)half, has(freq) ? f64(*freq, "freq") : nullptr, (float)mult,
                       r ? i32(*pos, T, "pos") : nullptr, dcode(x), stream()), "head_linear");
  return y;
}

// window: keys a token sees, itself included (0: all)
Tensor latent_generic(Tensor q, Tensor lat, Tensor bt, Tensor pos, Tensor seq_ids, int64_t R, double scale, OptT sink,
                      int64_t window) {
  need(q, "q"); table(bt, 1);
  const Lat c = lat_of(lat);
  const int64_t T = q.size(0), H = q.size(1);
  TORCH_CHECK(q.dim() == 3 && q.size(2) == c.W && q.scalar_type() == lat.scalar_type() && R > 0 && R <= c.W && window >= 0,
              "latent_generic: q");
  TORCH_CHECK(c.W <= 1024, "latent_generic: rows up to 1024");
  auto o = torch::empty({T, H, R}, q.options());
  check(ds_paged_generic(q.data_ptr(), lat.data_ptr(), lat.data_ptr(), o.data_ptr(), bt.data_ptr<int>(), (int)bt.size(1),
                         i32(pos, T, "pos"), i32(seq_ids, T, "seq_ids"), (int)T, (int)H, 1, c.W, (int)R, c.W, c.BS, (float)scale,
                         0.f, (int)window, 0, opt_f32(sink, H, "sink"), H * R, nullptr, 0, dcode(q), stream()), "latent_generic");
  return o;
}

bool latent_tiled_ok(int64_t d, int64_t r, int64_t e, int64_t R) {
  return ds_latent_decode_ok((int)R, (int)r) && ds_latent_prefill_ok((int)d, (int)r, (int)e);
}

// Tokens tok0 .. tok1 of the batch, those of sequences first .. first + nseq with up to max_new tokens each:
// q [.., H, R + r] -> out [.., H, R], rows tok0 .. tok1 of both
void latent_decode(Tensor q, Tensor lat, Tensor bt, Tensor cu, Tensor start, int64_t first, int64_t nseq, int64_t max_new,
                   int64_t tok0, int64_t tok1, int64_t max_len, int64_t R, double scale, OptT sink, Tensor out,
                   int64_t window) {
  need(q, "q"); need(out, "out"); table(bt, first + nseq);
  const Lat c = lat_of(lat);
  const int64_t H = q.size(1), n = tok1 - tok0, S = start.numel();
  TORCH_CHECK(q.dim() == 3 && q.size(2) == c.W && q.scalar_type() == at::kBFloat16 && lat.scalar_type() == at::kBFloat16 &&
              tok0 >= 0 && n >= 0 && tok1 <= q.size(0) && first >= 0 && first + nseq <= S && max_new > 0 &&
              bt.size(1) * c.BS >= max_len && ds_latent_decode_ok((int)R, (int)(c.W - R)), "latent_decode: q / latents / tables");
  TORCH_CHECK(out.dim() == 3 && out.size(0) >= tok1 && out.size(1) == H && out.size(2) == R && out.scalar_type() == q.scalar_type(),
              "latent_decode: out");
  int range = 0, splits = 1;
  TORCH_CHECK(window >= 0, "latent_decode: window");
  const int64_t span = window > 0 ? std::min(max_len, window + max_new - 1) : max_len;
  ds_latent_decode_plan((int)nseq, (int)max_new, (int)H, c.W, (int)span, &range, &splits);
  Tensor acc, ml;
  if (splits > 1) {
    auto fo = q.options().dtype(at::kFloat);
    acc = torch::empty({splits, n * H, R}, fo);
    ml = torch::empty({splits, n * H, 2}, fo);
  }
  check(ds_latent_decode((const char*)q.data_ptr() + tok0 * H * c.W * 2, lat.data_ptr(), (char*)out.data_ptr() + tok0 * H * R * 2,
                         splits > 1 ? acc.data_ptr<float>() : nullptr, splits > 1 ? ml.data_ptr<float>() : nullptr,
                         bt.data_ptr<int>(), (int)bt.size(1), i32(cu, S + 1, "cu"), i32(start, S, "start"), (int)first, (int)nseq,
                         (int)max_new, (int)tok0, (int)n, (int)H, (int)R, (int)(c.W - R), c.BS, range, splits,
                         (int)window, opt_f32(sink, H, "sink"), (float)scale, stream()), "latent_decode");
}

// cached rows of the contexts of sequences first .. first + nseq, from their first keys on, end to end, and PAD_ROWS rows of zeros: latent_prefill
// reads whole tiles of keys
constexpr int PAD_ROWS = 64;
const int* first_of(const OptT& t, int64_t n) { return has(t) ? i32(*t, n, "first keys") : nullptr; }
Tensor latent_gather(Tensor lat, Tensor bt, Tensor offs, OptT first_keys, int64_t first, int64_t total) {
  const Lat c = lat_of(lat);
  const int64_t nseq = offs.numel() - 1;
  table(bt, first + nseq);
  TORCH_CHECK(lat.scalar_type() == at::kBFloat16 && c.W % 8 == 0 && nseq > 0, "latent_gather: bf16 rows of 16-byte pieces");
  auto ctx = torch::empty({total + PAD_ROWS, c.W}, lat.options());
  check(ds_latent_gather(lat.data_ptr(), bt.data_ptr<int>(), (int)bt.size(1), i32(offs, nseq + 1, "offs"), first_of(first_keys, nseq), (int)first, (int)nseq,
                         ctx.data_ptr(), total, PAD_ROWS, c.W, c.BS, stream()), "latent_gather");
  return ctx;
}

// q [T, H, d + r] (tokens may lie further apart) rotated; kv [total + PAD_ROWS, H (d + e)], ctx [total + PAD_ROWS, R + r] -> rows of o [T, H, e] of the sequences in work
void latent_prefill(Tensor q, Tensor kv, Tensor ctx, Tensor start, Tensor cu_q, Tensor work, Tensor offs, OptT first_keys,
                    int64_t first, int64_t total, int64_t d, int64_t e, double scale, OptT sink, Tensor o, int64_t window) {
  const int64_t ldq = need_heads(q, "q");
  need(kv, "kv"); need(ctx, "ctx"); need(o, "o");
  const int64_t T = q.size(0), H = q.size(1), r = q.size(2) - d, S = start.numel();
  TORCH_CHECK(q.dim() == 3 && q.scalar_type() == at::kBFloat16 && kv.scalar_type() == at::kBFloat16 &&
              ctx.scalar_type() == at::kBFloat16 && kv.dim() == 2 && kv.size(1) == H * (d + e) && ctx.dim() == 2 &&
              ctx.size(0) == kv.size(0) && ctx.size(0) == total + PAD_ROWS && ctx.size(1) >= r && ds_latent_prefill_ok((int)d, (int)r, (int)e), "latent_prefill");
  TORCH_CHECK(o.dim() == 3 && o.size(0) == T && o.size(1) == H && o.size(2) == e && o.scalar_type() == q.scalar_type() &&
              work.dim() == 2 && work.size(1) == 2 && offs.numel() == S - first + 1 && scale > 0, "latent_prefill: o / tables");
  check(ds_latent_prefill(q.data_ptr(), kv.data_ptr(), ctx.data_ptr(), o.data_ptr(), i32(start, S, "start"),
                          i32(cu_q, S + 1, "cu_q"), i32(work, work.numel(), "work"), (int)work.size(0),
                          i32(offs, offs.numel(), "offs"), first_of(first_keys, S - first), (int)first, ldq, (int)window, (int)H, (int)d, (int)r, (int)e, (int)ctx.size(1),
                          (int)(ctx.size(1) - r), opt_f32(sink, H, "sink"), (float)scale, stream()), "latent_prefill");
}
}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("post_norm", &post_norm);
  m.def("gelu", &gelu);
  m.def("token_gate", &token_gate);
  m.def("latent_prepare", &latent_prepare);
  m.def("rotate_tail", &rotate_tail);
  m.def("head_linear", &head_linear, py::arg("x"), py::arg("w"), py::arg("freq") = py::none(), py::arg("pos") = py::none(),
        py::arg("out") = py::none(), py::arg("mult") = 1.0);
  m.def("latent_generic", &latent_generic);
  m.def("latent_tiled_ok", &latent_tiled_ok);
  m.def("latent_decode", &latent_decode);
  m.def("latent_gather", &latent_gather);
  m.def("latent_prefill", &latent_prefill);
}
