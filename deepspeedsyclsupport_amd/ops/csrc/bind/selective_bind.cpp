// Module of recurrences with a decay per channel and state, and of the short convolutions ahead of them. A shared object of its
// own, so that serving a model compiles the mechanisms it has and no others.
#include "bind_util.h"

extern "C" {
int ds_causal_conv(const void*, int64_t, const float*, const float*, void*, const int*, const int*, const int*, const int*,
                   void*, int, int, int, int, hipStream_t);
int ds_selective_scan_max();
int ds_selective_scan(const void*, const void*, const void*, int64_t, const void*, int64_t, const float*, const float*,
                      const float*, float*, const void*, int64_t, void*, const int*, int, int, const int*, const int*, const int*,
                      void*, int, int, int, int, int, int, hipStream_t);
}

namespace {
int64_t row_step(const Tensor& t) { return t.size(0) > 1 ? t.stride(0) : t.size(1); }
void window_ok(const OptT& cs, int64_t taps, int64_t C, const Tensor& x) {
  TORCH_CHECK(taps == 1 || (has(cs) && cs->is_cuda() && cs->is_contiguous() && cs->dim() == 3 && cs->size(1) == taps - 1 &&
              cs->size(2) == C && cs->scalar_type() == x.scalar_type()), "conv_state [slots, taps - 1, C]");
}

// x [T, C] (it may be columns of a wider matrix), w [C, taps], b [C] -> silu(conv(x) + b) [T, C]; the windows of portions of one
// token move on
Tensor causal_conv(Tensor x, Tensor w, Tensor b, OptT conv_state, Tensor seq_ids, Tensor cu, Tensor start, Tensor slots) {
  need_rows(x, "x");
  TORCH_CHECK(w.dim() == 2 && w.size(0) == x.size(1) && w.size(1) >= 1, "causal_conv: w [C, taps]");
  const int64_t T = x.size(0), C = x.size(1), taps = w.size(1), S = start.numel();
  window_ok(conv_state, taps, C, x);
  auto out = torch::empty({T, C}, x.options());
  check(ds_causal_conv(x.data_ptr(), row_step(x), f32(w, C * taps, "w"), f32(b, C, "b"), taps > 1 ? conv_state->data_ptr() : nullptr,
                       i32(seq_ids, T, "seq_ids"), i32(cu, S + 1, "cu"), i32(start, S, "start"), i32(slots, S, "slots"),
                       out.data_ptr(), (int)T, (int)C, (int)taps, dcode(x), stream()), "causal_conv");
  return out;
}

// Sequences of `list` ([n], or the first column of [n, 2]): x, dt [T, C], bc [T, 2 N], z [T, C] -> their rows of out [T, C]; their
// slots of state [slots, C, >= N] and, unless causal_conv has moved it on, conv_state (last rows of conv_x) advance. steps: few
// new tokens each
void selective_scan(Tensor x, Tensor dt, Tensor bc, Tensor z, Tensor dt_bias, Tensor decay, Tensor skip, Tensor state,
                    Tensor conv_x, OptT conv_state, Tensor list, Tensor cu, Tensor start, Tensor slots, bool steps, Tensor out) {
  need(x, "x"); need(dt, "dt"); need_rows(bc, "bc"); need_rows(z, "z"); need_rows(conv_x, "conv_x"); need(state, "state");
  need(out, "out");
  TORCH_CHECK(x.dim() == 2 && decay.dim() == 2, "selective_scan: x [T, C], decay [C, N]");
  const int64_t T = x.size(0), C = x.size(1), N = decay.size(1), S = start.numel(), L = list.size(0);
  auto like = [&](const Tensor& t, int64_t cols) {
    return t.dim() == 2 && t.size(0) == T && t.size(1) == cols && t.scalar_type() == x.scalar_type();
  };
  TORCH_CHECK(like(dt, C) && like(bc, 2 * N) && like(z, C) && like(conv_x, C) && like(out, C), "selective_scan: shapes / types");
  TORCH_CHECK(state.dim() == 3 && state.size(1) == C && state.size(2) >= N && state.scalar_type() == at::kFloat,
              "selective_scan: state [slots, C, N] fp32");
  TORCH_CHECK(N <= ds_selective_scan_max(), "selective_scan: up to ", ds_selective_scan_max(), " numbers per channel");
  const int64_t taps = has(conv_state) ? conv_state->size(1) + 1 : 1;
  window_ok(conv_state, taps, C, x);
  TORCH_CHECK(taps == 1 || conv_state->size(0) == state.size(0), "selective_scan: slots");
  check(ds_selective_scan(x.data_ptr(), dt.data_ptr(), bc.data_ptr(), row_step(bc), z.data_ptr(), row_step(z),
                          f32(dt_bias, C, "dt_bias"), f32(decay, C * N, "decay"), f32(skip, C, "skip"), state.data_ptr<float>(),
                          conv_x.data_ptr(), row_step(conv_x), taps > 1 ? conv_state->data_ptr() : nullptr,
                          i32(list, list.numel(), "list"), (int)L, L ? (int)(list.numel() / L) : 1, i32(cu, S + 1, "cu"),
                          i32(start, S, "start"), i32(slots, S, "slots"), out.data_ptr(), steps, (int)C, (int)N,
                          (int)state.size(2), (int)taps, dcode(x), stream()), "selective_scan");
}
}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("causal_conv", &causal_conv);
  m.def("selective_scan", &selective_scan);
}
