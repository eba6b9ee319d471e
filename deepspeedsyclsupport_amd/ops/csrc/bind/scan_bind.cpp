// Module of recurrences with a scalar decay per head and of the gated norms behind them: convolutions, rotations and gates ahead
// of the scan, the scan token by token and by chunks, with or without a normaliser. A shared object of its own, so that serving
// a model compiles the mechanisms it has and no others.
#include "bind_util.h"

extern "C" {
int ds_gated_norm(const void*, const void*, int64_t, const float*, void*, int64_t, int64_t, int, int, float, int, int,
                  hipStream_t);
int ds_scan_prepare(const void*, const float*, const float*, const void*, const float*, const float*, const int*, const int*,
                    const int*, const int*, void*, void*, float*, const int*, int, int, hipStream_t);
int ds_scan_split(const void*, const float*, int, void*, void*, int, const int*, int, int, hipStream_t);
int ds_exp_gates(const void*, int, int, int, const float*, const float*, float, float*, const int*, const int*, const int*,
                 float*, float*, int, int, int, int, hipStream_t);
int ds_scan_recur(const void*, const void*, const float*, const float*, const float*, float, const void*, float*, float*,
                  const float*, void*, int, const int*, int, int, const int*, const int*, const int*, void*, const int*, int,
                  int, hipStream_t);
int ds_scan_chunk_ok(int);
int ds_scan_chunk(const void*, const void*, const float*, const float*, const float*, float, const void*, float*, float*,
                  const float*, void*, int, const int*, int, const int*, const int*, const int*, void*, const int*, int,
                  hipStream_t);
}

namespace {
// y [T, C] with the gate columns proj[:, gate:gate + C] -> [T, C], into `out` (a matrix whose rows may be columns of wider ones)
// if there is one. mode: 0 norm, then sigmoid(gate); 1 silu(gate), then norm; 2 norm, then silu(gate)
Tensor gated_norm(Tensor y, Tensor proj, int64_t gate, OptT w, int64_t parts, double eps, int64_t mode, OptT out) {
  need(y, "y"); need(proj, "proj");
  const int64_t T = y.size(0), C = y.size(1);
  TORCH_CHECK(y.dim() == 2 && proj.dim() == 2 && proj.size(0) == T && gate >= 0 && gate + C <= proj.size(1) &&
              proj.scalar_type() == y.scalar_type() && parts > 0 && C % parts == 0, "gated_norm: y [T, C], gate columns of proj");
  Tensor o = has(out) ? *out : torch::empty_like(y);
  need_rows(o, "out");
  TORCH_CHECK(o.size(0) == T && o.size(1) == C && o.scalar_type() == y.scalar_type(), "gated_norm: out [T, C]");
  check(ds_gated_norm(y.data_ptr(), (const char*)proj.data_ptr() + gate * proj.element_size(), proj.size(1), opt_f32(w, C, "norm"),
                      o.data_ptr(), T > 1 ? o.stride(0) : C, T, (int)C, (int)parts, (float)eps, (int)mode, dcode(y), stream()),
        "gated_norm");
  return o;
}

// ---------------------------------------------------------------------------------------------- recurrences
struct Dims {  // ops/mixer_ops.py: ScanLayout
  int v[12];
  int rows() const { return v[0]; }
  int Hk() const { return v[4]; }
  int H() const { return v[5]; }
  int dk() const { return v[6]; }
  int dv() const { return v[7]; }
  int taps() const { return v[8]; }
  int conv() const { return v[9]; }
  int channels() const { return v[10]; }
  int dt() const { return v[11]; }
  int dks() const { return (dk() + 7) / 8 * 8; }
  int dvs() const { return (dv() + 7) / 8 * 8; }
};
Dims dims_of(const std::vector<int64_t>& d) {
  TORCH_CHECK(d.size() == 12, "scan: 12 dimensions");
  Dims D;
  for (int i = 0; i < 12; ++i) D.v[i] = (int)d[i];
  TORCH_CHECK(D.Hk() > 0 && D.H() > 0 && D.H() % D.Hk() == 0 && D.dk() > 0 && D.dk() <= 512 && D.dv() > 0 && D.taps() >= 1,
              "scan: head counts / sizes (keys up to 512)");
  auto inside = [&](int64_t at, int64_t n, int64_t lo, int64_t hi) { return at >= lo && at + n <= hi; };
  const int64_t nk = (int64_t)D.Hk() * D.dk(), nv = (int64_t)D.H() * D.dv(), lo = D.channels() ? D.conv() : 0,
                hi = D.channels() ? D.conv() + D.channels() : D.rows();
  TORCH_CHECK(inside(D.conv(), D.channels(), 0, D.rows()) && inside(D.v[1], nk, lo, hi) && inside(D.v[2], nk, lo, hi) &&
              inside(D.v[3], nv, lo, hi) && (D.dt() < 0 || inside(D.dt(), D.H(), 0, D.rows())) &&
              (D.taps() == 1 || D.channels() > 0), "scan: columns outside the projection");
  return D;
}
void conv_ok(const Dims& D, const OptT& cs, const Tensor& proj) {
  TORCH_CHECK(D.taps() == 1 || (has(cs) && cs->is_cuda() && cs->is_contiguous() && cs->dim() == 3 && cs->size(1) == D.taps() - 1 &&
              cs->size(2) == D.channels() && cs->scalar_type() == proj.scalar_type()), "scan: conv_state [slots, taps-1, channels]");
}

// proj [T, rows] -> qk [2, Hk, T, dks], v [H, T, dvs] (storage type), gb [T, 2, H] fp32 or None
std::tuple<Tensor, Tensor, OptT> scan_prepare(Tensor proj, std::vector<int64_t> dims, OptT conv_w, OptT conv_b, OptT conv_state,
                                              OptT a_log, OptT dt_bias, Tensor seq_ids, Tensor cu, Tensor start, Tensor slots) {
  need(proj, "proj");
  const Dims D = dims_of(dims);
  const int64_t T = proj.size(0), S = start.numel();
  TORCH_CHECK(proj.dim() == 2 && proj.size(1) == D.rows(), "scan_prepare: proj [T, rows]");
  TORCH_CHECK(has(conv_w) == (D.channels() > 0) && has(conv_b) == has(conv_w), "scan_prepare: convolution weights");
  conv_ok(D, conv_state, proj);
  // (rows are padded to 16-byte pieces with zeros)
  auto make = [&](at::IntArrayRef s, bool pad) { return pad ? torch::zeros(s, proj.options()) : torch::empty(s, proj.options()); };
  Tensor qk = make({2, D.Hk(), T, D.dks()}, D.dks() != D.dk()), v = make({D.H(), T, D.dvs()}, D.dvs() != D.dv());
  OptT gb;
  if (D.dt() >= 0) gb = torch::empty({T, 2, D.H()}, proj.options().dtype(at::kFloat));
  check(ds_scan_prepare(proj.data_ptr(), opt_f32(conv_w, (int64_t)D.channels() * D.taps(), "conv_w"),
                        opt_f32(conv_b, D.channels(), "conv_b"), D.taps() > 1 ? conv_state->data_ptr() : nullptr,
                        D.dt() >= 0 ? f32(*a_log, D.H(), "a_log") : nullptr, D.dt() >= 0 ? f32(*dt_bias, D.H(), "dt_bias") : nullptr,
                        i32(seq_ids, T, "seq_ids"), i32(cu, S + 1, "cu"), i32(start, S, "start"), i32(slots, S, "slots"),
                        qk.data_ptr(), v.data_ptr(), gb ? gb->data_ptr<float>() : nullptr, D.v, (int)T, dcode(proj), stream()),
        "scan_prepare");
  return {qk, v, gb};
}

// The same qk and v straight from the projection's columns, the first 2 half of every head of q and k turned by cs [T, half, 2];
// turned ones in bf16 as sums of two terms: qk [2 terms, 2, Hk, T, dks]
std::tuple<Tensor, Tensor> scan_split(Tensor proj, std::vector<int64_t> dims, OptT cs) {
  need(proj, "proj");
  const Dims D = dims_of(dims);
  const int64_t T = proj.size(0), half = has(cs) ? cs->numel() / 2 / std::max<int64_t>(T, 1) : 0;
  TORCH_CHECK(proj.dim() == 2 && proj.size(1) == D.rows() && 2 * half <= D.dk(), "scan_split: proj [T, rows]");
  auto make = [&](at::IntArrayRef s, bool pad) { return pad ? torch::zeros(s, proj.options()) : torch::empty(s, proj.options()); };
  const int terms = half > 0 && proj.scalar_type() == at::kBFloat16 ? 2 : 1;
  Tensor qk = make({terms, 2, D.Hk(), T, D.dks()}, D.dks() != D.dk()), v = make({D.H(), T, D.dvs()}, D.dvs() != D.dv());
  check(ds_scan_split(proj.data_ptr(), has(cs) ? f32(*cs, T * half * 2, "angles") : nullptr, (int)half, qk.data_ptr(), v.data_ptr(),
                      terms, D.v, (int)T, dcode(proj), stream()), "scan_split");
  return {qk, v};
}

// Columns ci .. ci + H, cf .. cf + H of proj [T, rows] -> gb [T, 2, H] (log decay, step size), floors [T, H]; peak [slots, H]
// advances
std::tuple<Tensor, Tensor> exp_gates(Tensor proj, int64_t ci, int64_t cf, Tensor bi, Tensor bf, double cap, Tensor peak, Tensor cu,
                                     Tensor start, Tensor slots, int64_t longest) {
  need(proj, "proj"); need(peak, "peak");
  const int64_t T = proj.size(0), H = bi.numel(), S = start.numel();
  TORCH_CHECK(proj.dim() == 2 && ci >= 0 && cf >= 0 && ci + H <= proj.size(1) && cf + H <= proj.size(1) && cap > 0,
              "exp_gates: columns outside the projection");
  TORCH_CHECK(peak.dim() == 2 && peak.size(1) == H && peak.scalar_type() == at::kFloat, "exp_gates: peak [slots, H] fp32");
  auto fo = proj.options().dtype(at::kFloat);
  Tensor gb = torch::empty({T, 2, H}, fo), floors = torch::empty({T, H}, fo);
  check(ds_exp_gates(proj.data_ptr(), (int)proj.size(1), (int)ci, (int)cf, f32(bi, H, "input bias"), f32(bf, H, "forget bias"),
                     (float)cap, peak.data_ptr<float>(), i32(cu, S + 1, "cu"), i32(start, S, "start"), i32(slots, S, "slots"),
                     gb.data_ptr<float>(), floors.data_ptr<float>(), (int)S, (int)longest, (int)H, dcode(proj), stream()),
        "exp_gates");
  return {gb, floors};
}

int terms_of(const Dims& D, const Tensor& qk, int64_t T) { return qk.numel() > 2 * D.Hk() * T * D.dks() ? 2 : 1; }

struct ScanCheck {
  ScanCheck(const Dims& D, const Tensor& qk, const Tensor& v, const OptT& gb, const OptT& ld, const Tensor& proj,
            const Tensor& state, const OptT& conv_state, const OptT& zstate, const OptT& floors, const Tensor& out) {
    need(qk, "qk"); need(v, "v"); need(proj, "proj"); need(state, "state"); need(out, "out");
    const int64_t T = proj.size(0);
    TORCH_CHECK(proj.size(1) == D.rows() && qk.numel() == terms_of(D, qk, T) * 2 * D.Hk() * T * D.dks() && v.numel() == D.H() * T * D.dvs() &&
                qk.scalar_type() == proj.scalar_type() && v.scalar_type() == proj.scalar_type(), "scan: qk / v");
    TORCH_CHECK(has(gb) != has(ld), "scan: decays per token or per head");
    TORCH_CHECK(state.scalar_type() == at::kFloat && state.dim() == 4 && state.size(1) == D.H() && state.size(2) == D.dv() &&
                state.size(3) == D.dks(), "scan: state [slots, H, dv, dks] fp32");
    TORCH_CHECK(out.numel() == T * D.H() * D.dv() && out.scalar_type() == proj.scalar_type(), "scan: out [T, H dv]");
    TORCH_CHECK(has(zstate) == has(floors), "scan: normaliser and floors");
    if (has(zstate)) {
      TORCH_CHECK(terms_of(D, qk, T) == 1, "scan: a normaliser takes q and k of one term");
      need(*zstate, "normaliser");
      TORCH_CHECK(zstate->scalar_type() == at::kFloat && zstate->dim() == 4 && zstate->size(0) == state.size(0) &&
                  zstate->size(1) == D.H() && zstate->size(2) == (D.dv() + 31) / 32 && zstate->size(3) == D.dks(),
                  "scan: normaliser [slots, H, dv / 32, dks] fp32");
    }
    conv_ok(D, conv_state, proj);
    TORCH_CHECK(D.taps() == 1 || conv_state->size(0) == state.size(0), "scan: slots");
  }
};

// Runs the sequences in `list` token by token; writes their rows of out and their state slots
void recur_list(Tensor qk, Tensor v, OptT gb, OptT log_decay, OptT skip, double scale, Tensor proj, const Dims& D,
                Tensor state, OptT zstate, OptT floors, OptT conv_state, Tensor list, int stride, Tensor cu, Tensor start, Tensor slots, Tensor out) {
  const int64_t T = proj.size(0), S = start.numel();
  check(ds_scan_recur(qk.data_ptr(), v.data_ptr(), opt_f32(gb, T * 2 * D.H(), "gb"), opt_f32(log_decay, D.H(), "log_decay"),
                      opt_f32(skip, D.H(), "skip"), (float)scale, proj.data_ptr(), state.data_ptr<float>(),
                      has(zstate) ? zstate->data_ptr<float>() : nullptr, opt_f32(floors, T * D.H(), "floors"),
                      D.taps() > 1 ? conv_state->data_ptr() : nullptr, terms_of(D, qk, T), i32(list, list.numel(), "list"),
                      (int)(list.numel() / stride), stride, i32(cu, S + 1, "cu"), i32(start, S, "start"), i32(slots, S, "slots"),
                      out.data_ptr(), D.v, (int)T, dcode(proj), stream()), "scan_recur");
}

void scan_recur(Tensor qk, Tensor v, OptT gb, OptT log_decay, OptT skip, double scale, Tensor proj,
                std::vector<int64_t> dims, Tensor state, OptT zstate, OptT floors, OptT conv_state, Tensor list, Tensor cu, Tensor start, Tensor slots, Tensor out) {
  const Dims D = dims_of(dims);
  ScanCheck(D, qk, v, gb, log_decay, proj, state, conv_state, zstate, floors, out);
  recur_list(qk, v, gb, log_decay, skip, scale, proj, D, state, zstate, floors, conv_state, list, 1, cu, start, slots, out);
}

// The same for long portions, seqs [n, 2]: bf16 by chunks of 64 tokens on the matrix cores; fp32 (and key widths above 256)
// token by token
void scan_chunk(Tensor qk, Tensor v, OptT gb, OptT log_decay, OptT skip, double scale, Tensor proj,
                std::vector<int64_t> dims, Tensor state, OptT zstate, OptT floors, OptT conv_state, Tensor seqs, Tensor cu, Tensor start, Tensor slots, Tensor out) {
  const Dims D = dims_of(dims);
  ScanCheck(D, qk, v, gb, log_decay, proj, state, conv_state, zstate, floors, out);
  TORCH_CHECK(seqs.dim() == 2 && seqs.size(1) == 2, "scan_chunk: seqs [n, 2]");
  if (proj.scalar_type() != at::kBFloat16 || !ds_scan_chunk_ok(D.dk())) {
    recur_list(qk, v, gb, log_decay, skip, scale, proj, D, state, zstate, floors, conv_state, seqs, 2, cu, start, slots, out);
    return;
  }
  const int64_t T = proj.size(0), S = start.numel();
  check(ds_scan_chunk(qk.data_ptr(), v.data_ptr(), opt_f32(gb, T * 2 * D.H(), "gb"), opt_f32(log_decay, D.H(), "log_decay"),
                      opt_f32(skip, D.H(), "skip"), (float)scale, proj.data_ptr(), state.data_ptr<float>(),
                      has(zstate) ? zstate->data_ptr<float>() : nullptr, opt_f32(floors, T * D.H(), "floors"),
                      D.taps() > 1 ? conv_state->data_ptr() : nullptr, terms_of(D, qk, T), i32(seqs, seqs.numel(), "seqs"), (int)seqs.size(0),
                      i32(cu, S + 1, "cu"), i32(start, S, "start"), i32(slots, S, "slots"), out.data_ptr(), D.v, (int)T, stream()),
        "scan_chunk");
}
}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("gated_norm", &gated_norm);
  m.def("scan_prepare", &scan_prepare);
  m.def("scan_split", &scan_split);
  m.def("exp_gates", &exp_gates);
  m.def("scan_recur", &scan_recur);
  m.def("scan_chunk", &scan_chunk);
}
