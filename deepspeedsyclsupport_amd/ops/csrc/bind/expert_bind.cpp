// Module of mixture-of-experts layers with grouped routing, and of the plain fp32 residual with RMS norms on the sublayers'
// inputs (and gated outputs), which takes the experts' weighted sum in the same pass. A shared object of its own, so that serving a model compiles
// the mechanisms it has and no others.
#include "bind_util.h"

extern "C" {
int ds_pre_norm(float*, const void*, const float*, const int*, const void*, int, const float*, const void*, int64_t, const float*,
                const int*, const void*, float, const int*, int, const float*, void*, int, float, int, hipStream_t);
int ds_route(const void*, const void*, int*, float*, int*, int*, int, int, int, int, int, int, int, int, float, int, hipStream_t);
int ds_expert_place(const int*, const int*, const int*, int*, int*, int*, int, int, hipStream_t);
int ds_expert_spread(const void*, const int*, void*, int, int, int64_t, hipStream_t);
int ds_expert_few();
int ds_expert_order_ok(int, int);
int ds_expert_gemm(const void*, const void*, void*, const int*, const int*, const int*, int, int, int, int, int, int, int, int,
                   int, hipStream_t);
int ds_expert_sum(const void*, const float*, const int*, const void*, void*, int, int, int, int, hipStream_t);
int ds_row_act(const void*, int64_t, void*, int64_t, int, int, int, hipStream_t);
}

namespace {
constexpr int SILU_GLU = 1, RELU2 = 2;  // activation codes

// x [T, W] fp32, in place: x += y [T, W], or x += sum_k yw[t, k] y[yrow[t, k]] + base (yrow none: row t K + k), or
// x = mult embed[ids]; what is added may be gated by sigmoid(gate + gate_b) and normed by post first. -> x / rms(x) w (w none: x)
// in y's / embed's type; with rows: those rows of it (x stays)
Tensor pre_norm(Tensor x, OptT y, OptT yw, OptT yrow, OptT base, OptT w, double eps, OptT ids, OptT embed, double mult, OptT rows,
                OptT post, OptT gate, OptT gate_b) {
  need(x, "x");
  TORCH_CHECK(x.scalar_type() == at::kFloat && x.dim() == 2, "pre_norm: x [T, W] fp32");
  const int64_t T = x.size(0), W = x.size(1);
  TORCH_CHECK(has(y) != has(embed) && !(has(rows) && has(embed)) && (!has(yw) || has(y)) && (!has(yrow) || has(yw)) &&
              (!has(base) || has(yw)), "pre_norm: y or embed");
  const Tensor& src = has(y) ? *y : *embed;
  need(src, "y / embed");
  const int64_t K = has(yw) ? yw->numel() / std::max<int64_t>(T, 1) : 1;
  TORCH_CHECK(src.dim() == 2 && src.size(1) == W && (has(embed) || src.size(0) == T * K), "pre_norm: y [T K, W]");
  if (has(base)) {
    need(*base, "base");
    TORCH_CHECK(base->dim() == 2 && base->size(0) == T && base->size(1) == W && base->scalar_type() == src.scalar_type(),
                "pre_norm: base [T, W]");
  }
  TORCH_CHECK(!has(post) || has(y), "pre_norm: a norm of what is added");
  if (has(gate)) {
    need_rows(*gate, "gate");
    TORCH_CHECK(has(post) && has(gate_b) && gate->size(0) == T && gate->size(1) == W && gate->scalar_type() == src.scalar_type(),
                "pre_norm: gate [T, W] with its bias and the norm behind it");
  }
  const int64_t R = has(rows) ? rows->numel() : T;
  auto out = torch::empty({R, W}, src.options());
  check(ds_pre_norm(x.data_ptr<float>(), has(y) ? y->data_ptr() : nullptr, opt_f32(yw, T * K, "weights"),
                    has(yrow) ? i32(*yrow, T * K, "y rows") : nullptr, has(base) ? base->data_ptr() : nullptr, (int)K,
                    opt_f32(post, W, "post norm"), has(gate) ? gate->data_ptr() : nullptr,
                    has(gate) && T > 1 ? gate->stride(0) : W, has(gate) ? f32(*gate_b, W, "gate bias") : nullptr,
                    has(embed) ? i32(*ids, T, "ids") : nullptr, has(embed) ? embed->data_ptr() : nullptr, (float)mult,
                    has(rows) ? i32(*rows, R, "rows") : nullptr, (int)R, opt_f32(w, W, "norm weight"), out.data_ptr(), (int)W,
                    (float)eps, dcode(src), stream()), "pre_norm");
  return out;
}

// h [T, W], router [E, W] -> experts int32 [T, K], weights fp32 [T, K], and with `lists` offs [E + 1], order [T K], rows [T, K]
// score: 0 softmax over all experts, 1 sigmoids; best: members that count for a group
std::tuple<Tensor, Tensor, OptT, OptT, OptT> route(Tensor h, Tensor router, int64_t K, int64_t groups, int64_t keep, bool lists,
                                                   int64_t score, int64_t best, double scale) {
  need(h, "h"); need(router, "router");
  TORCH_CHECK(h.dim() == 2 && router.dim() == 2 && h.size(1) == router.size(1) && h.scalar_type() == router.scalar_type(),
              "route: h [T, W], router [E, W]");
  const int64_t T = h.size(0), W = h.size(1), E = router.size(0);
  TORCH_CHECK(E >= 1 && E <= 256 && K >= 1 && K <= 64, "route: up to 256 experts, 64 of them at a time");
  TORCH_CHECK(groups >= 1 && E % groups == 0 && keep >= 1 && keep <= groups && K <= keep * (E / groups), "route: groups");
  TORCH_CHECK(T * K <= INT32_MAX / 2, "route: tokens");
  TORCH_CHECK((score == 0 || score == 1) && (best == 1 || best == 2), "route: softmax or sigmoid, one or two members of a group");
  auto io = h.options().dtype(at::kInt);
  auto experts = torch::empty({T, K}, io), weights = torch::empty({T, K}, h.options().dtype(at::kFloat));
  OptT offs, order, rows;
  Tensor counts, slots;
  if (lists) {
    counts = torch::zeros({E}, io);
    slots = torch::empty({T, K}, io);
  }
  check(ds_route(h.data_ptr(), router.data_ptr(), experts.data_ptr<int>(), weights.data_ptr<float>(),
                 lists ? counts.data_ptr<int>() : nullptr, lists ? slots.data_ptr<int>() : nullptr, (int)T, (int)W, (int)E, (int)K,
                 (int)groups, (int)keep, (int)score, (int)best, (float)scale, dcode(h), stream()), "route");
  if (lists) {
    offs = torch::empty({E + 1}, io);
    order = torch::empty({T * K}, io);
    rows = torch::empty({T, K}, io);
    check(ds_expert_place(experts.data_ptr<int>(), slots.data_ptr<int>(), counts.data_ptr<int>(), offs->data_ptr<int>(),
                          order->data_ptr<int>(), rows->data_ptr<int>(), (int)(T * K), (int)E, stream()), "expert_place");
  }
  return {experts, weights, offs, order, rows};
}

// x [T, W] -> [T K, W] with row rows[t, k] = x[t]
Tensor expert_spread(Tensor x, Tensor rows) {
  need(x, "x");
  const int64_t T = x.size(0), W = x.size(1), K = rows.size(-1);
  TORCH_CHECK(x.dim() == 2 && W * x.element_size() % 16 == 0, "expert_spread: rows of whole 16-byte pieces");
  auto out = torch::empty({T * K, W}, x.options());
  check(ds_expert_spread(x.data_ptr(), i32(rows, T * K, "rows"), out.data_ptr(), (int)T, (int)K, W * x.element_size(), stream()),
        "expert_spread");
  return out;
}

int64_t expert_few() { return ds_expert_few(); }

bool expert_order_ok(int64_t N, int64_t K) { return ds_expert_order_ok((int)N, (int)K); }

// x [rows, K], w [E, N or 2 N, K], experts [entries] -> y [entries, N]: y[i] = w[experts[i]] x[i / div]; act 1: silu(first N
// rows) times the last N; 2: max(., 0)^2. offs, order: lists from `route`. operand: the elements of w are in operand order; tile: many rows per
// expert (operand order and lists only)
Tensor expert_gemm(Tensor x, Tensor w, Tensor experts, OptT offs, OptT order, int64_t div, int64_t act, bool operand, bool tile) {
  need(x, "x"); need(w, "w");
  const bool gated = act == SILU_GLU;
  const int64_t entries = experts.numel(), E = w.size(0), K = w.size(2), N = w.size(1) / (gated ? 2 : 1);
  TORCH_CHECK(x.dim() == 2 && w.dim() == 3 && x.size(1) == K && x.scalar_type() == w.scalar_type() && E <= 256 &&
              (!gated || w.size(1) % 2 == 0) && div > 0 && entries % div == 0 && x.size(0) == entries / div, "expert_gemm: shapes");
  TORCH_CHECK(has(offs) == has(order), "expert_gemm: lists");
  auto y = torch::empty({entries, N}, x.options());
  check(ds_expert_gemm(x.data_ptr(), w.data_ptr(), y.data_ptr(), i32(experts, entries, "experts"),
                       has(offs) ? i32(*offs, E + 1, "offs") : nullptr, has(order) ? i32(*order, entries, "order") : nullptr,
                       (int)entries, (int)E, (int)N, (int)K, (int)div, (int)act, operand, tile, dcode(x), stream()), "expert_gemm");
  return y;
}

// y [T K, W], weights [T, K] -> sum_k weights[t, k] y[rows[t, k]] (rows none: t K + k), plus base [T, W]
Tensor expert_sum(Tensor y, Tensor w, OptT rows, OptT base) {
  need(y, "y");
  const int64_t T = w.size(0), K = w.size(1), W = y.size(1);
  TORCH_CHECK(y.dim() == 2 && w.dim() == 2 && y.size(0) == T * K, "expert_sum: y [T K, W]");
  if (has(base)) {
    need(*base, "base");
    TORCH_CHECK(base->numel() == T * W && base->scalar_type() == y.scalar_type(), "expert_sum: base [T, W]");
  }
  auto out = torch::empty({T, W}, y.options());
  check(ds_expert_sum(y.data_ptr(), f32(w, T * K, "weights"), has(rows) ? i32(*rows, T * K, "rows") : nullptr,
                      has(base) ? base->data_ptr() : nullptr, out.data_ptr(), (int)T, (int)W, (int)K, dcode(y), stream()), "expert_sum");
  return out;
}

// Rows [R, F] that may be columns of wider ones; act 1: [R, gate | up] -> silu(gate) up; 2: max(x, 0)^2
Tensor row_act(Tensor x, int64_t act) {
  need_rows(x, "x");
  TORCH_CHECK((act == SILU_GLU && x.size(1) % 2 == 0) || act == RELU2, "row_act: [R, gate | up], or any rows");
  const int64_t R = x.size(0), F = x.size(1) / (act == SILU_GLU ? 2 : 1);
  auto out = torch::empty({R, F}, x.options());
  check(ds_row_act(x.data_ptr(), R > 1 ? x.stride(0) : x.size(1), out.data_ptr(), R, (int)F, (int)act, dcode(x), stream()),
        "row_act");
  return out;
}
}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("pre_norm", &pre_norm);
  m.def("route", &route, py::arg("h"), py::arg("router"), py::arg("top"), py::arg("groups"), py::arg("keep"), py::arg("lists"),
        py::arg("score") = 0, py::arg("best") = 1, py::arg("scale") = 1.0);
  m.def("expert_spread", &expert_spread);
  m.def("expert_few", &expert_few);
  m.def("expert_order_ok", &expert_order_ok);
  m.def("expert_gemm", &expert_gemm);
  m.def("expert_sum", &expert_sum);
  m.def("row_act", &row_act);
}
