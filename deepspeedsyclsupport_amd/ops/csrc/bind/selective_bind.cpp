// Module of recurrences with a decay per channel and state, and of the short convolutions ahead of them. A shared object of its
// own, so that serving a model compiles the mechanisms it has and no others.
#include "bind_util.h"

extern "C" {
int ds_causal_conv(const void*, int64_t, const float*, const float*, const void*, const int*, const int*, const int*, const int*,
                   void*, int, int, int, int, hipStream_t);
int ds_selective_scan_max();
int ds_selective_scan(const void*, const void*, const void*, int64_t, const void*, int64_t, const float*, const float*,
                      const float*, float*, const void*, int64_t, void*, const int*, const int*, const int*, void*, int, int, int,
                      int, int, int, int, hipStream_t);
}

namespace {
int64_t row_step(const Tensor& t) { return t.size(0) > 1 ? t.stride(0) : t.size(1); }
void window_ok(const OptT& cs, int64_t taps, int64_t C, const Tensor& x) {
  TORCH_CHECK(taps == 1 || (has(cs) && cs->is_cuda() && cs->is_contiguous() && cs->dim() == 3 && cs->size(1) == taps - 1 &&
              cs->size(2) == C && cs->scalar_type() == x.scalar_type()), "conv_state [slots, taps - 1, C]");
}

// x [T, C] (it may be columns of a wider matrix), w [C, taps], b [C] -> silu(conv(x) + b) [T, C]
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

// x, dt [T, C], bc [T, 2 N], z [T, C] -> out [T, C]; state [slots, C, >= N] and conv_state (last rows of conv_x) advance
Tensor selective_scan(Tensor x, Tensor dt, Tensor bc, Tensor z, Tensor dt_bias, Tensor a_log, Tensor skip, Tensor state,
                      Tensor conv_x, OptT conv_state, Tensor cu, Tensor start, Tensor slots) {
  need(x, "x"); need(dt, "dt"); need_rows(bc, "bc"); need_rows(z, "z"); need_rows(conv_x, "conv_x"); need(state, "state");
  TORCH_CHECK(x.dim() == 2 && a_log.dim() == 2, "selective_scan: x [T, C], a_log [C, N]");
  const int64_t T = x.size(0), C = x.size(1), N = a_log.size(1), S = start.numel();
  auto like = [&](const Tensor& t, int64_t cols) { return t.size(0) == T && t.size(1) == cols && t.scalar_type() == x.scalar_type(); };
  TORCH_CHECK(dt.dim() == 2 && like(dt, C) && like(bc, 2 * N) && like(z, C) && like(conv_x, C), "selective_scan: shapes / types");
  TORCH_CHECK(state.dim() == 3 && state.size(1) == C && state.size(2) >= N && state.scalar_type() == at::kFloat,
              "selective_scan: state [slots, C, N] fp32");
  TORCH_CHECK(N <= ds_selective_scan_max(), "selective_scan: up to ", ds_selective_scan_max(), " numbers per channel");
  const int64_t taps = has(conv_state) ? conv_state->size(1) + 1 : 1;
  window_ok(conv_state, taps, C, x);
  TORCH_CHECK(taps == 1 || conv_state->size(0) == state.size(0), "selective_scan: slots");
  auto out = torch::empty({T, C}, x.options());
  check(ds_selective_scan(x.data_ptr(), dt.data_ptr(), bc.data_ptr(), row_step(bc), z.data_ptr(), row_step(z),
                          f32(dt_bias, C, "dt_bias"), f32(a_log, C * N, "a_log"), f32(skip, C, "skip"), state.data_ptr<float>(),
                          conv_x.data_ptr(), row_step(conv_x), taps > 1 ? conv_state->data_ptr() : nullptr, i32(cu, S + 1, "cu"),
                          i32(start, S, "start"), i32(slots, S, "slots"), out.data_ptr(), (int)S, (int)((T + S - 1) / S), (int)C,
                          (int)N, (int)state.size(2), (int)taps, dcode(x), stream()), "selective_scan");
  return out;
}
}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("causal_conv", &causal_conv);
  m.def("selective_scan", &selective_scan);
}
