"""Ops of the hybrid decoder (`inference/model_implementations/hybrid.py`): multi-stream residual, attention with
per-head norms and chunked visibility, gated delta rule, clamped gated activation.

Device tensors run the gfx950 kernels of `ds_hybrid_ops`, `ds_attn_ops` and `ds_gemv_ops` (fp32 or bf16 storage, fp32
arithmetic); host tensors the plain versions in `ops/reference.py`, as everywhere in `ops`."""
import torch
import torch.nn.functional as F

from . import mixer_ops, reference
from .native import attn_ops, gemv_ops, hybrid_ops, use_native

DECODE_ROWS = 16
ACTS = {"gelu": 2}  # epilogue codes of the decode products (csrc/gemv/skinny_*.hip)


def stream_norm(x, y, mix, out, m, in_, w, eps, ids=None, embed=None, rows=None):
    """Finish a sublayer (y, mix, out) or embed (ids, embed) into the streams x [T, S, W] fp32, in place, and return
    the layer norm of sum_s in_[s] x_s. `rows`: norm these rows only and leave x as it is (in_ None: plain sum)."""
    f = hybrid_ops().stream_norm if use_native(x) else reference.stream_norm
    return f(x, y, mix, out, m, in_, w, eps, ids, embed, rows)


def clamped_glu(gu, limit, alpha=1.702, shift=1.0):
    """[.., gate | up] -> g sigmoid(alpha g) (u + shift) with g = min(gate, limit), u = clamp(up, +-limit)."""
    f = hybrid_ops().clamped_glu if use_native(gu) else reference.clamped_glu
    return f(gu, limit, alpha, shift)


def qk_norm_append(qkv, qw, kw, eps, vfirst, lam, pos, seq_ids, block_table, kc, vc, H, cs=None):
    """Rows [q | k | v] (they may be columns of wider ones) -> q [T, H, dk]; k and v into the paged cache. The pairs (2 i, 2 i + 1)
    of every query and key head's first 2 half columns are turned by cs [T, half, 2] (None: no rotation), then each head is
    divided by its root mean square, times qw / kw (None: no weight)."""
    f = attn_ops().qk_norm_append if use_native(qkv) else reference.qk_norm_append
    return f(qkv, qw, kw, eps, vfirst, lam, pos, seq_ids, block_table, kc, vc, H, cs)


def rope_table(pos, freq, mult=1.0):
    """cos and sin of pos [T] * freq [half] (fp64), times `mult` -> [T, half, 2] fp32."""
    return (attn_ops() if use_native(pos) else reference).rope_table(pos, freq, mult)


def qk_rope_append(qkv, bias, qw, kw, eps, cs, meta, kc, vc, H, v_mult=1.0):
    """Rows [q | k | v] (they may be columns of wider ones) plus bias -> q [T, H, dk]; k, and v times `v_mult`, into the paged
    cache. q and k are divided by the root mean square over all their heads, times qw / kw (None: no norm), then the pairs
    (i, i + half) of every head's first 2 half columns are turned by cs [T, half, 2] (None: no rotation)."""
    f = attn_ops().qk_rope_append if use_native(qkv) else reference.qk_rope_append
    return f(qkv, bias, qw, kw, eps, cs, v_mult, meta.pos_ids, meta.seq_ids, meta.block_tables, kc, vc, H)


def ragged_attention(q, kc, vc, meta, scale, softcap=0.0, window=0, chunk=0, sink=None, out=None, gate=None):
    """q [T, H, dk] of a ragged batch (`RaggedMeta`) over the paged cache, the new tokens already appended -> [T, H, dv], or
    into `out` [T, H dv] (it may be columns of a wider matrix). `sink` [H]: exp(sink) joins the denominators. `gate` [T, H]
    (columns of a wider matrix): every head's output times the sigmoid of its number."""
    T, H, dv = q.shape[0], q.shape[1], vc.shape[3]
    args = (meta.block_tables, meta.pos_ids, meta.seq_ids, scale, softcap, window, chunk)
    if out is None:
        out = q.new_empty(T, H * dv)
        return ragged_attention(q, kc, vc, meta, scale, softcap, window, chunk, sink, out, gate).view(T, H, dv)
    if not use_native(q):
        return out.copy_(reference.paged_attention(q, kc, vc, *args, sink, gate).reshape(T, H * dv))
    ops = attn_ops()
    if q.dtype != torch.bfloat16 or not ops.paged_tiled_ok(kc.shape[3], dv):
        return ops.paged_generic(q, kc, vc, *args, sink, out, gate)
    nd = meta.n_decode
    if nd < len(meta.start_host):
        ops.paged_prefill(q, kc, vc, meta.block_tables, meta.start_pos, meta.cu_q, meta.work, scale, softcap, window, chunk,
                          sink, out, gate)
    if nd:
        ops.paged_decode(q[:nd], kc, vc, meta.block_tables[:nd], meta.seq_lens[:nd], meta.max_len, scale, softcap, window,
                         chunk, out, sink, gate)
    return out


def delta_rule(proj, conv_w, a_log, dt_bias, norm_w, eps, state, conv_state, meta, Hk, H, dk, dv):
    """Fused projection rows [T, q | k | v | g | b | a] -> gated, normed read-out [T, H dv]; the state slots advance."""
    out = proj.new_empty(proj.shape[0], H * dv)
    ops = hybrid_ops() if use_native(proj) else reference
    qk, v, gb = ops.delta_prepare(proj, conv_w, conv_state, a_log, dt_bias, meta.seq_ids, meta.cu_q, meta.start_pos,
                                  meta.slots, Hk, H, dk, dv)
    if meta.seq_list.numel():
        ops.delta_recur(qk, v, gb, proj, norm_w, eps, state, conv_state, meta.seq_list, meta.cu_q, meta.start_pos,
                        meta.slots, out, dk)
    if meta.chunk_work.numel():
        ops.delta_chunk(qk, v, gb, proj, norm_w, eps, state, conv_state, meta.chunk_seqs, meta.chunk_work, meta.cu_q,
                        meta.start_pos, meta.slots, out, dk)
    return out


def linear(x, w, sh=None, act=None):
    """x . w^T: a weight stream for decode-sized bf16 batches (over the shuffled copy `sh`, a `Bf16Weight`, from two
    rows up), else the library product. act "gelu": the exact gelu of it (the stream's epilogue, else a pass of its own)."""
    rows = x.numel() // x.shape[-1]
    code = None if act is None else ACTS[act]
    if sh is not None and x.is_cuda and x.is_contiguous() and 2 <= rows <= DECODE_ROWS:
        return gemv_ops().decode_linear_sh(x, sh.wsh, sh.shape[0], act=code)
    if x.is_cuda and x.is_contiguous() and x.dtype == torch.bfloat16 and 0 < rows <= DECODE_ROWS and \
            gemv_ops().decode_linear_ok(rows, x.shape[-1]):
        return gemv_ops().decode_linear(x, w, act=code)
    y = F.linear(x, w)
    return y if act is None else mixer_ops.gelu(y)


def glu_linear(x, w, sh, limit):
    """Clamped gated activation of x . [gate | up]^T: the epilogue of the weight stream for decode-sized bf16 batches."""
    rows = x.numel() // x.shape[-1]
    if x.is_cuda and x.dtype == torch.bfloat16 and 0 < rows <= DECODE_ROWS:
        if sh is not None and rows >= 2:
            return gemv_ops().decode_linear_sh(x, sh.wsh, sh.shape[0], limit)
        if gemv_ops().decode_linear_ok(rows, x.shape[-1]):
            return gemv_ops().decode_linear(x, w, limit)
    return clamped_glu(F.linear(x, w), limit)
