"""Ops of decoders with routed experts (`inference/model_implementations/hybrid.py`): one fp32 residual with RMS norms on the
sublayers' inputs and, optionally, on their gated outputs, grouped routing, expert products.

Device tensors run the gfx950 kernels of `ds_expert_ops` (fp32 or bf16 storage); host tensors the plain versions in
`ops/reference.py`, as everywhere in `ops`. Residual, norms, router logits and scores are fp32 whatever the storage type."""
from dataclasses import dataclass
from typing import Optional

import torch

from . import reference
from .native import expert_ops, use_native


@dataclass
class ExpertSum:
    """A sublayer's output not yet summed: token t adds sum_k w[t, k] y[rows[t, k]] (rows None: row t K + k), and base[t]."""
    y: torch.Tensor
    w: torch.Tensor
    rows: Optional[torch.Tensor] = None
    base: Optional[torch.Tensor] = None

    def sum(self):
        """The plain tensor [T, W]."""
        return (expert_ops() if use_native(self.y) else reference).expert_sum(self.y, self.w, self.rows, self.base)


def pre_norm(x, y, w, eps, ids=None, embed=None, mult=1.0, rows=None, post_w=None, gate=None, gate_b=None):
    """Residual x [T, W] fp32, in place: x += y (a tensor or an `ExpertSum`), or x = mult embed[ids]. Returns x / rms(x) * w (w
    None: x) in y's (embed's) type. With `rows`: x stays, and those rows come back. What is added may first be multiplied by
    sigmoid(gate + gate_b), gate [T, W] (it may be columns of a wider matrix), and then be divided by its own rms, times
    post_w."""
    f = (expert_ops() if use_native(x) else reference).pre_norm
    parts = (y.y, y.w, y.rows, y.base) if isinstance(y, ExpertSum) else (y, None, None, None)
    return f(x, *parts, w, eps, ids, embed, mult, rows, post_w, gate, gate_b)


ACTS = {"none": 0, "silu_glu": 1, "relu2": 2}   # of a product's rows; silu_glu: silu(first half) times the second
SCORES = {"softmax": 0, "sigmoid": 1}


def row_act(x, act):
    """An activation of rows [R, F] ([R, gate | up] for a gated one); they may be columns of wider ones."""
    return (expert_ops() if use_native(x) else reference).row_act(x, ACTS[act])


# Average rows per expert from which on the products tile the rows instead of streaming the weights (in operand order)
TILE_ROWS = 12
# ... and, where only row-major weights are kept, go to the library's grouped GEMM over rows copied into expert order
LIBRARY_ROWS = 32


def operand_order(w):
    """Expert weights [E, N, K] as the products on the matrix cores read them (`bf16_gemv.preshuffle16` of every expert), or None
    where sizes or type do not allow it. N: rows of one expert (gate and up count as one half each)."""
    from .bf16_gemv import preshuffle16
    E, N, K = w.shape
    if w.dtype != torch.bfloat16 or not w.is_cuda or not expert_ops().expert_order_ok(N, K):
        return None
    return torch.stack([preshuffle16(e) for e in w]).view(E, N, K)


def experts(h, router, fc1, fc2, top, groups=1, keep=1, order=None, score="softmax", best=1, scale=1.0, act="silu_glu"):
    """Routed feed-forwards: h [T, W], router [E, W], fc1 [E, F, W] (gated: [E, 2 F, W], gate rows, up rows), fc2 [E, W, F] ->
    `ExpertSum`. Experts are scored by the softmax over all or by their own sigmoids. Those of the `keep` best of `groups` equal
    groups compete (a group counts as much as its `best` best members together); the `top` best are taken, weighted by their
    scores divided by the scores' sum, times `scale`. `order`: (fc1, fc2) in operand order, if they are kept."""
    code, routing = ACTS[act], (top, groups, keep)
    how = (SCORES[score], best, scale)
    if not use_native(h):
        e, w = reference.route(h, router, *routing, *how)
        return ExpertSum(reference.expert_gemm(reference.expert_gemm(h, fc1, e, top, code), fc2, e, 1, 0), w)
    ops = expert_ops()
    rows, E = h.shape[0] * top, router.shape[0]
    tile = order is not None and rows >= TILE_ROWS * E
    few = h.dtype != torch.bfloat16 or (rows <= ops.expert_few() and not tile)
    e, w, offs, entries, at = ops.route(h, router, *routing, not few, *how)
    if order is None and not few and rows >= LIBRARY_ROWS * E and all(n % 128 == 0 for n in (*fc1.shape[1:], fc2.shape[2])):
        ends = offs[1:]
        mid = ops.row_act(torch._grouped_mm(ops.expert_spread(h, at), fc1.transpose(1, 2), offs=ends), code)
        return ExpertSum(torch._grouped_mm(mid, fc2.transpose(1, 2), offs=ends), w, at)
    (a, b), operand = (order, True) if order else ((fc1, fc2), False)
    mid = ops.expert_gemm(h, a, e, offs, entries, top, code, operand, tile)
    return ExpertSum(ops.expert_gemm(mid, b, e, offs, entries, 1, 0, operand, tile), w)
