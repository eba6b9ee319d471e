"""Ops of pre-norm decoders with routed experts (`inference/model_implementations/hybrid.py`): plain fp32 residual with RMS
norms on the sublayers' inputs, grouped routing, expert products.

Device tensors run the gfx950 kernels of `ds_expert_ops` (fp32 or bf16 storage); host tensors the plain versions in
`ops/reference.py`, as everywhere in `ops`. Residual, norms, router logits and scores are fp32 whatever the storage type."""
from dataclasses import dataclass
from typing import Optional

import torch

from . import reference
from .native import expert_ops, use_native


@dataclass
class ExpertSum:
    """A sublayer's output not yet summed: token t adds sum_k w[t, k] y[rows[t, k]] (rows None: row t K + k)."""
    y: torch.Tensor
    w: torch.Tensor
    rows: Optional[torch.Tensor] = None

    def sum(self):
        """The plain tensor [T, W]."""
        return (expert_ops() if use_native(self.y) else reference).expert_sum(self.y, self.w, self.rows)


def pre_norm(x, y, w, eps, ids=None, embed=None, mult=1.0, rows=None):
    """Residual x [T, W] fp32, in place: x += y (a tensor or an `ExpertSum`), or x = mult embed[ids]. Returns x / rms(x) * w in
    y's (embed's) type. With `rows`: x stays, and those rows come back."""
    f = (expert_ops() if use_native(x) else reference).pre_norm
    if isinstance(y, ExpertSum):
        return f(x, y.y, y.w, y.rows, w, eps, ids, embed, mult, rows)
    return f(x, y, None, None, w, eps, ids, embed, mult, rows)


# From this many rows on the products go to the library's grouped GEMM, over rows copied into expert order
LIBRARY_ROWS = 1024


def experts(h, router, fc1, fc2, top, groups=1, keep=1):
    """Routed gated feed-forwards: h [T, W], router [E, W], fc1 [E, 2 F, W] (gate rows, up rows), fc2 [E, W, F] -> `ExpertSum`.
    The experts of the `keep` best of `groups` equal groups compete; the best `top` are taken, weighted by their softmax over
    all experts divided by its sum."""
    if not use_native(h):
        e, w = reference.route(h, router, top, groups, keep)
        return ExpertSum(reference.expert_gemm(reference.expert_gemm(h, fc1, e, top, True), fc2, e, 1, False), w)
    ops = expert_ops()
    rows = h.shape[0] * top
    few = rows <= ops.expert_few() or h.dtype != torch.bfloat16
    e, w, offs, order, at = ops.route(h, router, top, groups, keep, not few)
    if rows >= LIBRARY_ROWS and not few and all(n % 128 == 0 for n in (*fc1.shape[1:], fc2.shape[2])):
        ends = offs[1:]
        mid = ops.silu_mul(torch._grouped_mm(ops.expert_spread(h, at), fc1.transpose(1, 2), offs=ends))
        return ExpertSum(torch._grouped_mm(mid, fc2.transpose(1, 2), offs=ends), w, at)
    mid = ops.expert_gemm(h, fc1, e, offs, order, top, True)
    return ExpertSum(ops.expert_gemm(mid, fc2, e, offs, order, 1, False), w)
