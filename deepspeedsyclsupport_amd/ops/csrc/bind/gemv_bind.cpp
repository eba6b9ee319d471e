// Module of the bf16 decode products (up to 16 token rows) of the hybrid decoders, with activation epilogues.
#include "bind_util.h"

#include <map>
#include <utility>

extern "C" {
int ds_skinny_gemm(const void*, const void*, const void*, const void*, const void*, const void*, void*, void*, int, int,
                   int, int, int, int, float, hipStream_t);
int ds_skinny_b16_mfma_ok(int, int);
int ds_skinny_b16_mfma(const void*, const void*, const void*, void*, float*, int, int, int, hipStream_t);
int ds_skinny_finalize_gated(float*, const void*, void*, int, int, int, int, float, hipStream_t);
int ds_skinny_mfma_ok(int, int, int);
int ds_skinny_mfma(const void*, const void*, const void*, const void*, const void*, const void*, void*, void*, int, int,
                   int, int, int, int, float, hipStream_t);
int ds_skinny_finalize_act(float*, void*, int, int, int, int, hipStream_t);
}

namespace {
bool decode_linear_ok(int64_t M, int64_t K) {
  return M >= 1 && K % 8 == 0 && (M <= 8 || (M <= 16 && ds_skinny_mfma_ok((int)M, (int)K, 0)));
}
constexpr int CLAMPED_GLU = 5;  // DS_ACT_CLAMPED_GLU
constexpr int UNARY = 16;       // DS_ACT_UNARY

// x [M, K] . w [N, K]^T for M <= 16 bf16 rows: the vector kernel up to two rows (or where K does not tile), else MFMA.
// act: an activation code applied to the result. With a limit instead, w is a fused [gate | up] weight and the result its
// clamped gated activation [M, N / 2].
Tensor decode_linear(Tensor x, Tensor w, std::optional<double> glu_limit, std::optional<int64_t> act) {
  need(x, "x"); need(w, "w");
  const int64_t N = w.size(0), K = w.size(1), M = x.numel() / K;
  const bool glu = glu_limit.has_value();
  TORCH_CHECK(x.scalar_type() == at::kBFloat16 && w.scalar_type() == at::kBFloat16 && x.size(-1) == K, "decode_linear");
  TORCH_CHECK(decode_linear_ok(M, K), "decode_linear: up to 8 rows with K % 8 == 0 (16 with K % 256 == 0)");
  TORCH_CHECK(!glu || N % 2 == 0, "decode_linear: [gate | up] rows");
  auto sizes = x.sizes().vec();
  sizes.back() = glu ? N / 2 : N;
  auto y = torch::empty(sizes, x.options());
  TORCH_CHECK(!(glu && act.has_value()), "decode_linear: one epilogue");
  const int code = glu ? CLAMPED_GLU : act.has_value() ? UNARY + (int)*act : 0;
  auto fn = M > 2 && ds_skinny_mfma_ok((int)M, (int)K, 0) ? ds_skinny_mfma : ds_skinny_gemm;
  check(fn(w.data_ptr(), x.data_ptr(), nullptr, nullptr, nullptr, nullptr, y.data_ptr(), nullptr, (int)M, (int)N, (int)K,
           0, glu ? 1 : 0, code, glu ? (float)*glu_limit : 0.f, stream()), "decode_linear");
  return y;
}

// The same over a weight in the shuffled decode layout (ops/bf16_gemv.py: preshuffle16), w [N, K], K % 64 == 0
Tensor decode_linear_sh(Tensor x, Tensor wsh, int64_t N, std::optional<double> glu_limit, std::optional<int64_t> act) {
  need(x, "x"); need(wsh, "wsh");
  const int64_t K = x.size(-1), M = x.numel() / K, NB = (N + 15) / 16;
  const bool glu = glu_limit.has_value();
  TORCH_CHECK(x.scalar_type() == at::kBFloat16 && wsh.scalar_type() == at::kBFloat16 && wsh.numel() == NB * 16 * K &&
              ds_skinny_b16_mfma_ok((int)M, (int)K), "decode_linear_sh: up to 16 bf16 rows, K % 64 == 0");
  TORCH_CHECK(NB * K < ((int64_t)1 << 40) && N < ((int64_t)1 << 31) / 16, "decode_linear_sh: matrix too large");
  TORCH_CHECK(!(glu && act.has_value()), "decode_linear_sh: one epilogue");
  TORCH_CHECK(!glu || N % 2 == 0, "decode_linear_sh: [gate | up] rows");
  // fp32 split-K sums, zero between calls (the kernels leave it so); one per device and stream, grown on demand
  static std::map<std::pair<int, hipStream_t>, Tensor> workspaces;
  Tensor& ws = workspaces[{x.get_device(), stream()}];
  const int64_t NP = (NB + 3) / 4 * 64;  // row length of the sums
  if (!ws.defined() || ws.numel() < 16 * NP) ws = torch::zeros({16 * NP}, x.options().dtype(at::kFloat));
  auto sizes = x.sizes().vec();
  sizes.back() = glu ? N / 2 : N;
  auto y = torch::empty(sizes, x.options());
  check(ds_skinny_b16_mfma(x.data_ptr(), wsh.data_ptr(), nullptr, glu || act.has_value() ? nullptr : y.data_ptr(),
                           ws.data_ptr<float>(), (int)M, (int)N, (int)K, stream()), "decode_linear_sh");
  if (act.has_value())
    check(ds_skinny_finalize_act(ws.data_ptr<float>(), y.data_ptr(), (int)M, (int)N, (int)NP, (int)*act, stream()),
          "decode_linear_sh (activation)");
  if (glu)
    check(ds_skinny_finalize_gated(ws.data_ptr<float>(), nullptr, y.data_ptr(), (int)M, (int)N, (int)NP, CLAMPED_GLU,
                                   (float)*glu_limit, stream()), "decode_linear_sh (gated)");
  return y;
}
}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("decode_linear", &decode_linear, py::arg("x"), py::arg("w"), py::arg("glu_limit") = py::none(),
        py::arg("act") = py::none());
  m.def("decode_linear_ok", &decode_linear_ok);
  m.def("decode_linear_sh", &decode_linear_sh, py::arg("x"), py::arg("wsh"), py::arg("N"),
        py::arg("glu_limit") = py::none(), py::arg("act") = py::none());
}
