"""Ops of hybrid decoders without residual streams (`inference/model_implementations/hybrid.py`): norms on sublayer
outputs, latent attention, recurrences with a scalar decay per head or a decay per channel and state, gated norms, token-side
inputs.

Device tensors run the gfx950 kernels of `ds_mixer_ops`, `ds_scan_ops` and `ds_selective_ops` (fp32 or bf16 storage); host tensors the plain
versions in `ops/reference.py`, as everywhere in `ops`. Residual, norms, angles, scores, softmax, decays and the recurrent state are
fp32 whatever the storage type."""
from dataclasses import dataclass

import torch
import torch.nn.functional as F

from . import reference
from .native import mixer_ops, scan_ops, selective_ops, use_native


def post_norm(x, y, w, eps, ids=None, embed=None, rows=None, final_w=None, mult=1.0):
    """Residual x [T, W] fp32, in place: x += y / rms(y) * w, or x = embed[ids]. Returns x in y's (embed's) type, the
    next sublayer's input. With `rows`: x stays, and those rows of the sum come back RMS-normed by `final_w`, times
    `mult`."""
    f = mixer_ops().post_norm if use_native(x) else reference.post_norm
    return f(x, y, w, eps, ids, embed, rows, final_w, mult)


def gelu(x):
    """Exact gelu."""
    return mixer_ops().gelu(x) if use_native(x) else reference.gelu_erf(x)


def token_gate(g, ids, table, first):
    """gelu_tanh(g) * table[ids, first:first + width]."""
    f = mixer_ops().token_gate if use_native(g) else reference.token_gate
    return f(g, ids, table, first)


GATES = {"sigmoid_after": 0, "silu_before": 1, "silu_after": 2}


def gated_norm(y, proj, gate, w, parts, eps, mode, out=None):
    """y [T, C] with the gate columns proj[:, gate:gate + C]: every one of `parts` equal parts of a row by its own rms, times w
    (None: no weight), times sigmoid(gate) or silu(gate); "silu_before": silu(gate) comes before the norm. `out`: where to
    write (a matrix that may be columns of a wider one)."""
    f = scan_ops().gated_norm if use_native(y) else reference.gated_norm
    return f(y, proj, gate, w, parts, eps, GATES[mode], out)


# ------------------------------------------------------------------------------------------------ latent attention
def latent_prepare(down, qw, kvw, eps, freq, meta, lat, q_rank, mult=1.0):
    """Projection rows [q latent | kv latent | rotated part] (they may be columns of wider ones) -> normed query latent
    [T, q_rank] (q_rank 0: None); the normed latent and the rotated part of every token go into the paged cache lat
    [blocks, 1, block, kv_rank + rot]. `mult`: factor of cosine and sine."""
    f = mixer_ops().latent_prepare if use_native(down) else reference.latent_prepare
    return f(down, qw, kvw, eps, freq, mult, meta.pos_ids, meta.seq_ids, meta.block_tables, lat, q_rank)


def latent_attention(q, lat, ukv, ukt, freq, sink, meta, scale, d, e, window=0, mult=1.0):
    """q [T, H, d + rot] (not rotated yet; tokens may lie further apart) of a ragged batch over the paged latents -> [T, H, e].
    `sink` [H] (or None): exp(sink) joins the denominators. `window`: keys a token sees, itself included (0: all before it).

    Decodes and short portions fold the key map into the query and attend to the latents themselves (every cached byte is
    read once for all heads); longer portions expand keys and values of their context (what the window lets their first token
    see of it, and on) with one product and run tiled attention per head. ukv [H (d + e), kv_rank]: key rows, then value rows;
    ukt [H, kv_rank, d]: the key map per head."""
    T, H, R = q.shape[0], q.shape[1], ukt.shape[1]
    if not use_native(q):
        return reference.latent_attention(q, lat, ukv, freq, mult, sink, meta.block_tables, meta.pos_ids, meta.seq_ids, scale, d,
                                          e, window)
    ops = mixer_ops()
    tiled = q.dtype == torch.bfloat16 and ops.latent_tiled_ok(d, q.shape[2] - d, e, R)
    short = meta.cu_host[meta.n_short] if tiled else T
    o = q.new_empty(T, H, e)
    if short:
        ql = ops.head_linear(q[:short], ukt, freq, meta.pos_ids[:short], None, mult)  # [short, H, R + rot]
        if tiled:
            ol = q.new_empty(short, H, R)
            cu = meta.cu_host
            for a, b in ((0, meta.n_decode), (meta.n_decode, meta.n_short)):  # decodes; short portions
                if a < b:
                    longest = 1 if b == meta.n_decode else max(cu[i + 1] - cu[i] for i in range(a, b))
                    ops.latent_decode(ql, lat, meta.block_tables, meta.cu_q, meta.start_pos, a, b - a, longest, cu[a], cu[b],
                                      meta.max_len, R, scale, sink, ol, window)
        else:
            ol = ops.latent_generic(ql, lat, meta.block_tables, meta.pos_ids, meta.seq_ids, R, scale, sink, window)
        ops.head_linear(ol, ukv[H * d:].view(H, e, R), out=o[:short])
    if short < T:
        offs, first_keys, total = meta.contexts(window)
        ctx = ops.latent_gather(lat, meta.block_tables, offs, first_keys, meta.n_short, total)
        kv = F.linear(ctx[:, :R], ukv)
        ops.rotate_tail(q[short:], freq, meta.pos_ids[short:], q.shape[2] - d, mult)
        ops.latent_prefill(q, kv, ctx, meta.start_pos, meta.cu_q, meta.work[meta.n_short - meta.n_decode:], offs, first_keys,
                           meta.n_short, total, d, e, scale, sink, o, window)
    return o


# ------------------------------------------------------------------------------------------------ recurrences
@dataclass(frozen=True)
class ScanLayout:
    """Where a fused projection row [rows] holds what. q, k [Hk heads of dk], v [H heads of dv] and the output gate start
    at the given columns. With taps > 1, columns conv .. conv + channels (they hold q, k and v) pass a causal convolution
    with bias. dt: first of H step-size columns, or -1 (decays and steps from elsewhere)."""
    rows: int
    q: int
    k: int
    v: int
    gate: int
    Hk: int
    H: int
    dk: int
    dv: int
    taps: int = 1
    conv: int = 0
    channels: int = 0
    dt: int = -1

    @property
    def dks(self):
        """Key width as the state is stored."""
        return -(-self.dk // 8) * 8


    @property
    def dims(self):
        return (self.rows, self.q, self.k, self.v, self.Hk, self.H, self.dk, self.dv, self.taps, self.conv, self.channels,
                self.dt)


def _scan(ops, proj, lay, qk, v, gb, log_decay, skip, scale, state, zstate, floors, conv_state, meta):
    out = proj.new_empty(proj.shape[0], lay.H * lay.dv)
    args = (qk, v, gb, log_decay, skip, scale, proj, lay.dims, state, zstate, floors, conv_state)
    if meta.seq_list.numel():
        ops.scan_recur(*args, meta.seq_list, meta.cu_q, meta.start_pos, meta.slots, out)
    if meta.chunk_seqs.numel():
        ops.scan_chunk(*args, meta.chunk_seqs, meta.cu_q, meta.start_pos, meta.slots, out)
    return out


def decayed_scan(proj, lay, state, meta, conv_w=None, conv_b=None, conv_state=None, a_log=None, dt_bias=None, skip=None,
                 log_decay=None):
    """S_t = a_t S_(t-1) + b_t k_t v_t^T, o_t = S_t^T q_t + skip v_t for every head -> [T, H dv]; state slots
    [slots, H, dv, dks] fp32 (and the convolution's windows) advance. q, k and v pass silu. Step sizes b = softplus(dt +
    dt_bias) with a = exp(-exp(a_log) b), or b = 1 with a = exp(log_decay).

    Portions up to `RaggedMeta.STEP_TOKENS` go token by token, longer ones by chunks."""
    ops = scan_ops() if use_native(proj) else reference
    qk, v, gb = ops.scan_prepare(proj, lay.dims, conv_w, conv_b, conv_state, a_log, dt_bias, meta.seq_ids, meta.cu_q,
                                 meta.start_pos, meta.slots)
    return _scan(ops, proj, lay, qk, v, gb, log_decay, skip, 1.0, state, None, None, conv_state, meta)


def retention(proj, lay, state, meta, log_decay, cs, scale):
    """S_t = exp(log_decay) S_(t-1) + k_t v_t^T, o_t = scale S_t^T q_t; the pairs (i, i + half) of every head's first 2 half
    columns of q and k are turned by cs [T, half, 2] (None: no rotation)."""
    ops = scan_ops() if use_native(proj) else reference
    qk, v = ops.scan_split(proj, lay.dims, cs)
    return _scan(ops, proj, lay, qk, v, None, log_decay, None, scale, state, None, None, None, meta)


def matrix_memory(proj, lay, slots, meta, gates, bi, bf, cap, scale):
    """Exponentially gated recurrence with a normaliser. Gate columns gates, gates + H of the projection give, per head,
    i = cap tanh((x + bi) / cap) and f = logsigmoid(cap tanh((x + bf) / cap)); m_t = max(f + m_(t-1), i) from m = 0, and
    S_t = e^(f + m_(t-1) - m_t) S_(t-1) + e^(i - m_t) k v^T, z likewise with k alone, o = c S^T q / (max(|c z . q|, e^-m) + 1e-6)
    with c = `scale`. `slots`: {"state": [.., H, dv, dks], "norm": [.., H, ceil(dv / 32), dks], "peak": [.., H]}."""
    ops = scan_ops() if use_native(proj) else reference
    cu = meta.cu_host
    longest = max(b - a for a, b in zip(cu, cu[1:]))
    gb, floors = ops.exp_gates(proj, gates, gates + lay.H, bi, bf, cap, slots["peak"], meta.cu_q, meta.start_pos, meta.slots,
                               longest)
    qk, v = ops.scan_split(proj, lay.dims, None)
    return _scan(ops, proj, lay, qk, v, gb, None, None, scale, slots["state"], slots["norm"], floors, None, meta)


# ------------------------------------------------------------------------------------------------ selective recurrences
def causal_conv(x, w, b, conv_state, meta):
    """silu(conv(x) + b): x [T, C] (it may be columns of a wider matrix), w [C, taps] (last column: the current token), inputs
    before a portion from its slot of conv_state [slots, taps - 1, C]. This op or the `selective_scan` that must follow moves the
    slots on, whichever does it more cheaply."""
    f = (selective_ops() if use_native(x) else reference).causal_conv
    return f(x, w, b, conv_state, *((meta.seq_ids, ) if use_native(x) else ()), meta.cu_q, meta.start_pos, meta.slots)


def selective_scan(x, dt, bc, z, dt_bias, decay, skip, state, conv_x, conv_state, meta):
    """A decay per channel and state: with step = softplus(dt + dt_bias) and decay [C, N] < 0,
    S[c, n] <- exp(step_c decay[c, n]) S[c, n] + step_c x_c B_n, y_c = sum_n S[c, n] C_n + skip_c x_c, out = y silu(z) [T, C]. bc
    [T, B | C], z [T, C]: columns of wider matrices. state [slots, C, N rounded up to 4] fp32 and conv_state, the last inputs
    of the convolution conv_x [T, C], advance.

    Portions up to `RaggedMeta.STEP_TOKENS` stream the state token by token, longer ones keep it in registers."""
    ops, out = selective_ops() if use_native(x) else reference, torch.empty_like(x)
    args = (x, dt, bc, z, dt_bias, decay, skip, state, conv_x, conv_state)
    for seqs, steps in ((meta.seq_list, True), (meta.chunk_seqs, False)):
        if seqs.numel():
            ops.selective_scan(*args, seqs, meta.cu_q, meta.start_pos, meta.slots, steps, out)
    return out
