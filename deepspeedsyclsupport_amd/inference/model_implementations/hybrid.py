"""Decoders whose layers differ from one another: every layer names its mixer (attention or a recurrence), the
mixer's sizes and its feed-forward (`DSModelSpec.layer_specs`), and the residual may run in several streams.

`DSHybridModel` is a `DSInferenceModel`: the engines, the ragged batch, the paged cache, sampling, quantisation and
serialisation treat it like any other. What is different sits in one class per mechanism, each with its sizes and
constants as parameters:

* `StreamResidual`    S fp32 residual streams, mixed by small matrices around every sublayer, fused with the pre-norm
* `PostNormResidual`  one fp32 residual; the sublayers read it as it is and their outputs are RMS-normed before the sum
* `PreNormResidual`   one fp32 residual with RMS norms on the sublayers' inputs
* `SandwichResidual`  one fp32 residual with RMS norms on the sublayers' inputs and outputs, and optionally a gate on the outputs
* `AttentionMixer`    GQA, key and value widths of their own, per-head query / key RMS norm, score cap, chunked
                      visibility, value mixing with an earlier layer; K / V live in the blocked cache
* `LatentMixer`       attention over a shared low-rank latent with a rotated key part, optionally with a query latent, a softmax
                      sink and a sliding window; only the latent and that key part are cached
* `DeltaMixer`        gated delta rule behind short convolutions; its fp32 state lives in a slot per sequence
* `Mamba2Mixer`       state-space recurrence with a scalar decay per head and token behind a short convolution
* `LightningMixer`    linear attention with a constant decay per head
* `RotaryAttention`   GQA with projection biases, query / key norms over all heads, partial rotation, chunked visibility and a
                      softmax sink
* `WindowAttention`   GQA over a sliding window, queries and keys rotated and then normed head by head, a gate per head
* `Mamba1Mixer`       selective state space: a decay per channel and state, behind a short convolution
* `MatrixMemory`      recurrence with exponential input and forget gates, a running maximum and a normaliser
* `Retention`         linear attention with rotated queries and keys and a constant decay per head
* `ParallelMixer`     two of these on the same input, their weighted outputs summed
* `ClampedMLP`        gated feed-forward with clamped gate and up branches
* `GatedMLP`          gated (silu) feed-forward
* `GeluMLP`           plain feed-forward with the exact gelu
* `RoutedMLP`         experts, chosen per token among the best groups of experts, optionally beside one that every token takes
* `TokenSide`         a small embedding per layer and token, gated by the residual

Per sublayer the launches are: residual + norm, one fused input projection, the mixer's kernels, the output projection.
"""
import math

import torch
import torch.nn as nn

from ...ops import expert_ops
from ...ops import hybrid_ops as ops
from ...ops import mixer_ops, op_builder
from .transformer import DSInferenceModel, ProjectionLayer


def _f32(shape, fill, device):
    return nn.Parameter(torch.full(shape, fill, dtype=torch.float32, device=device), requires_grad=False)


def _empty(shape, dtype, device):
    return nn.Parameter(torch.empty(*shape, dtype=dtype, device=device), requires_grad=False)


def _shard(t, r, tp, dim=0):
    return t if tp == 1 else t.chunk(tp, dim)[r]


def _up8(n):
    return -(-n // 8) * 8


def _fill_rows(w, rows, name):
    """w [rows, ..] with rows of zeros up to a multiple of 8."""
    if w.shape[0] != rows:
        raise ValueError(f"{name} has {w.shape[0]} rows in the checkpoint, {rows} by the configuration")
    return torch.cat([w, w.new_zeros(_up8(rows) - rows, *w.shape[1:])])


class StreamResidual(nn.Module):
    """Mixing weights of one sublayer: in_ [S], mix [S from, S to], out [S] (identity for a plain residual)."""

    extensions = ("ds_hybrid_ops", )

    def __init__(self, spec, device, side=False):
        super().__init__()
        streams, width = spec.streams, spec.hidden_size
        self.norm_w = _f32((width, ), 1.0, device)
        self.in_ = _f32((streams, ), 1.0, device)
        self.out = _f32((streams, ), 1.0, device)
        self.mix = _f32((streams, streams), 1.0, device)

    @staticmethod
    def begin(model, ids):
        """Residual of a batch and the first sublayer's input."""
        spec, first = model.spec, model.layers[0].res1
        x = torch.empty(ids.numel(), spec.streams, spec.hidden_size, dtype=torch.float32, device=model.embed.device)
        return x, ops.stream_norm(x, None, None, None, 1.0, first.in_, first.norm_w, spec.norm_eps, ids=ids,
                                  embed=model.embed)

    def enter(self, spec, x, pending):
        """Close the sublayer before (its output and residual weights) and norm this one's input."""
        y, prev, _ = pending
        return ops.stream_norm(x, y, prev.mix, prev.out, spec.residual_mult, self.in_, self.norm_w, spec.norm_eps)

    def finish(self, model, x, y, rows, gate=None):
        """Normed output rows of the model; this is the last sublayer's residual."""
        return ops.stream_norm(x, y, self.mix, self.out, model.spec.residual_mult, None, model.norm_w,
                               model.spec.norm_eps, rows=rows)

    def peek(self, spec, x, y, gate=None):
        """Sum of the streams after this sublayer."""
        return (torch.einsum("st,nsw->ntw", self.mix, x) +
                spec.residual_mult * self.out[None, :, None] * y[:, None].float()).sum(1)


class PostNormResidual(nn.Module):
    """Norm weight of one sublayer's output: x <- x + y / rms(y) * w."""

    extensions = ("ds_mixer_ops", )

    def __init__(self, spec, device, side=False):
        super().__init__()
        self.norm_w = _f32((spec.hidden_size, ), 1.0, device)

    @staticmethod
    def begin(model, ids):
        x = torch.empty(ids.numel(), model.spec.hidden_size, dtype=torch.float32, device=model.embed.device)
        return x, mixer_ops.post_norm(x, None, None, 0.0, ids=ids, embed=model.embed)

    def enter(self, spec, x, pending):
        y, prev, _ = pending
        return mixer_ops.post_norm(x, y, prev.norm_w, spec.norm_eps)

    def finish(self, model, x, y, rows, gate=None):
        return mixer_ops.post_norm(x, y, self.norm_w, model.spec.norm_eps, rows=rows, final_w=model.norm_w,
                                   mult=model.spec.logit_scale)

    def peek(self, spec, x, y, gate=None):
        y = y.float()
        return x + y * torch.rsqrt(y.pow(2).mean(-1, keepdim=True) + spec.norm_eps) * self.norm_w


class PreNormResidual(nn.Module):
    """Norm weight of one sublayer's input: x <- x + f(x / rms(x) * w). A sublayer may hand over an `ExpertSum`; it is summed
    in the pass that adds it."""

    extensions = ("ds_expert_ops", )

    def __init__(self, spec, device, side=False):
        super().__init__()
        self.norm_w = _f32((spec.hidden_size, ), 1.0, device)

    @staticmethod
    def begin(model, ids):
        spec = model.spec
        x = torch.empty(ids.numel(), spec.hidden_size, dtype=torch.float32, device=model.embed.device)
        return x, expert_ops.pre_norm(x, None, model.layers[0].res1.norm_w, spec.norm_eps, ids=ids, embed=model.embed,
                                      mult=spec.embed_scale)

    def enter(self, spec, x, pending):
        return expert_ops.pre_norm(x, pending[0], self.norm_w, spec.norm_eps)

    def finish(self, model, x, y, rows, gate=None):
        return expert_ops.pre_norm(x, y, model.norm_w, model.spec.norm_eps, rows=rows)

    def peek(self, spec, x, y, gate=None):
        return x + (y.sum() if isinstance(y, expert_ops.ExpertSum) else y).float()


class SandwichResidual(PreNormResidual):
    """Norm weights of one sublayer's input and output: x <- x + g / rms(g) * post_w with g = sigmoid(gate + gate_b) * f(h),
    h = x / rms(x) * norm_w; without `spec.residual_gate`, g = f(h). The gate is a linear map of h. `side`: a sublayer that reads x
    as it is, without a gate."""

    def __init__(self, spec, device, side=False):
        super().__init__(spec, device)
        self.side = side
        if side:
            del self.norm_w
        self.post_w = _f32((spec.hidden_size, ), 1.0, device)
        if spec.residual_gate and not side:
            self.gate_b = _f32((spec.hidden_size, ), 0.0, device)

    def _close(self, gate):
        """How `pre_norm` takes this sublayer's output."""
        return dict(post_w=self.post_w, gate=gate, gate_b=None if gate is None else self.gate_b)

    def enter(self, spec, x, pending):
        y, prev, gate = pending
        return expert_ops.pre_norm(x, y, None if self.side else self.norm_w, spec.norm_eps, **prev._close(gate))

    def finish(self, model, x, y, rows, gate=None):
        return expert_ops.pre_norm(x, y, model.norm_w, model.spec.norm_eps, rows=rows, **self._close(gate))

    def peek(self, spec, x, y, gate=None):
        y = (y.sum() if isinstance(y, expert_ops.ExpertSum) else y).float()
        if gate is not None:
            y = y * torch.sigmoid(gate.float() + self.gate_b)
        return x + y * torch.rsqrt(y.pow(2).mean(-1, keepdim=True) + spec.norm_eps) * self.post_w


RESIDUALS = {"streams": StreamResidual, "post_norm": PostNormResidual, "pre_norm": PreNormResidual, "sandwich": SandwichResidual}


class Mixer:
    """What a mixer may leave at its default. `rows`: width of the fused input projection; `out_width`: of its output."""
    extra_projections = ()   # names of weight matrices beside the input and output projection
    strided = False          # takes projection rows that are columns of wider ones
    extensions = ()          # native extensions its ops come from

    def parameters(self, device):
        """Small fp32 weights, by name."""
        return {}

    def matrices(self, dtype, device):
        """Weight matrices beside the input and output projection."""
        return {}

    def constants(self, device):
        """Tensors made from the configuration."""
        return {}

    def kv_geometry(self):
        """(heads, key width, value width) of the layer's cache, or None."""
        return None

    def state_geometry(self, dtype):
        """{name: (shape, dtype)} of the state a sequence carries, or None."""
        return None


class AttentionMixer(Mixer):
    """Sizes and constants of an attention mixer; the weights are the layer's."""
    kind = "attention"
    extensions = ("ds_hybrid_ops", "ds_attn_ops")

    def __init__(self, mx, tp):
        self.H, self.G, self.dk, self.dv = mx["heads"] // tp, mx["kv_heads"] // tp, mx["dim"], mx["vdim"]
        if mx["heads"] % mx["kv_heads"] or mx["kv_heads"] % tp:
            raise ValueError(f"{mx['heads']} query / {mx['kv_heads']} key heads over {tp} ranks")
        self.scale = float(mx["scale"])
        self.softcap = float(mx.get("softcap") or 0.0)
        self.chunk = int((mx.get("mask") or {}).get("size") or 0)
        self.v_mix = bool(mx.get("v_mix"))
        self.rows = (self.H + self.G) * self.dk + self.G * self.dv
        self.out_width = self.H * self.dv

    def parameters(self, device):
        p = {"q_norm": _f32((self.dk, ), 1.0, device), "k_norm": _f32((self.dk, ), 1.0, device)}
        if self.v_mix:
            p["vmix"] = _f32((1, ), 0.0, device)
        return p

    def shard(self, lw, r, tp):
        out = {"qkv_w": torch.cat([_shard(lw[n], r, tp) for n in ("q_w", "k_w", "v_w")]), "o_w": _shard(lw["o_w"], r, tp, 1),
               "q_norm": lw["q_norm"], "k_norm": lw["k_norm"]}
        if self.v_mix and "vmix" in lw:
            out["vmix"] = lw["vmix"].reshape(1)
        return out

    def kv_geometry(self):
        return self.G, self.dk, self.dv

    def run(self, layer, h, meta, cache, carry):
        qkv = layer.project(h, carry)
        kc, vc = cache.k[layer.layer_idx], cache.v[layer.layer_idx]
        v_first = None
        if self.v_mix:  # the first mixing layer lends its values to the later ones of the same step
            v_first = carry.get("v_first")
            if v_first is None:
                carry["v_first"] = qkv[:, (self.H + self.G) * self.dk:]
        q = ops.qk_norm_append(qkv, layer.q_norm, layer.k_norm, layer.spec.norm_eps, v_first,
                               layer.vmix if v_first is not None else None, meta.pos_ids, meta.seq_ids,
                               meta.block_tables, kc, vc, self.H)
        o = ops.ragged_attention(q, kc, vc, meta, self.scale, self.softcap, 0, self.chunk)
        return o.reshape(h.shape[0], self.out_width)


class DeltaMixer(Mixer):
    """Sizes of a gated-delta-rule mixer; the weights are the layer's."""
    kind = "delta"
    extensions = ("ds_hybrid_ops", )

    def __init__(self, mx, tp):
        if mx["heads"] % mx["kv_heads"] or mx["kv_heads"] % tp:
            raise ValueError(f"{mx['heads']} value / {mx['kv_heads']} key heads over {tp} ranks")
        self.H, self.Hk, self.dk, self.dv = mx["heads"] // tp, mx["kv_heads"] // tp, mx["dim"], mx["vdim"]
        self.taps = int(mx["conv"])
        self.channels = 2 * self.Hk * self.dk + self.H * self.dv
        self.rows = self.channels + self.H * self.dv + 2 * self.H
        self.out_width = self.H * self.dv

    def parameters(self, device):
        return {"conv_w": _f32((self.channels, self.taps), 0.0, device), "a_log": _f32((self.H, ), 0.0, device),
                "dt_bias": _f32((self.H, ), 0.0, device), "head_norm": _f32((self.dv, ), 1.0, device)}

    def shard(self, lw, r, tp):
        def s(n):
            return _shard(lw[n], r, tp)

        return {"qkv_w": torch.cat([s(n) for n in ("q_w", "k_w", "v_w", "g_w", "b_w", "a_w")]),
                "conv_w": torch.cat([s(n) for n in ("q_conv", "k_conv", "v_conv")]),
                "o_w": _shard(lw["o_w"], r, tp, 1), "a_log": s("a_log"), "dt_bias": s("dt_bias"),
                "head_norm": lw["head_norm"]}

    def state_geometry(self, dtype):
        return {"state": ((self.H, self.dv, -(-self.dk // 4) * 4), torch.float32), "conv": ((self.taps - 1, self.channels),
                                                                                         dtype)}

    def run(self, layer, h, meta, cache, carry):
        proj = layer.project(h, carry)
        st = cache.state[layer.layer_idx]
        return ops.delta_rule(proj, layer.conv_w, layer.a_log, layer.dt_bias, layer.head_norm, layer.spec.norm_eps,
                              st["state"], st["conv"], meta, self.Hk, self.H, self.dk, self.dv)


class Rotation:
    """Frequencies of rotated positions: pair i of `dims` / 2 turns by position * base^(-2 i / dims), slowed down by a scaling:

    * "linear": all by `factor`
    * "yarn": pairs that turn less than `slow` times within `original` positions by `factor`, those that turn more than `fast`
      times not at all, with a linear ramp between; cosine and sine grow by `mult`

    Pair i is columns (i, i + dims / 2); "neighbours": (2 i, 2 i + 1). The batch's angle table is made once per step for all
    layers with the same constants."""

    def __init__(self, rot, width):
        self.dims, self.base, self.neighbours = int(rot["dims"]), float(rot["base"]), rot.get("pairs") == "neighbours"
        scaling = rot.get("scaling") or {}
        self.factor, self.kind = float(scaling.get("factor", 1.0)), scaling.get("type", "linear")
        if self.dims % 2 or not 0 <= self.dims <= width:
            raise ValueError(f"{self.dims} rotated of {width} dimensions")
        if self.kind not in ("linear", "yarn"):
            raise NotImplementedError(f"no scaling {self.kind!r} of rotated positions")
        self.mult, self.key = 1.0, (self.dims, self.base, self.factor)
        if self.kind == "yarn":
            self.original, self.turns = float(scaling["original"]), (float(scaling["fast"]), float(scaling["slow"]))
            self.mult = 0.1 * math.log(self.factor) + 1.0
            self.key += (self.original, *self.turns)

    def _pair_of(self, turns):
        """The (fractional) pair that turns so many times within the original length."""
        return self.dims * math.log(self.original / (2 * math.pi * turns)) / (2 * math.log(self.base))

    def frequencies(self, device):
        i = torch.arange(self.dims // 2, dtype=torch.float64)
        f = self.base**(-2 * i / max(self.dims, 1))
        if self.kind == "linear":
            return (f / self.factor).to(device)
        lo, hi = max(math.floor(self._pair_of(self.turns[0])), 0), min(math.ceil(self._pair_of(self.turns[1])), self.dims - 1)
        ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0, 1)
        return (f / self.factor * ramp + f * (1 - ramp)).to(device)

    def halves(self, w, first=0):
        """Rows `first` .. of every head of w [heads, rows, ..] reordered so that pairs of neighbours become (i, i + dims / 2):
        scores do not see an order that queries and keys share."""
        if not self.neighbours:
            return w
        i = torch.arange(self.dims // 2)
        at = torch.cat([torch.arange(first), first + 2 * i, first + 2 * i + 1, torch.arange(first + self.dims, w.shape[1])])
        return w[:, at]

    def angles(self, freq, meta, carry):
        if not self.dims:
            return None
        tables = carry.setdefault("angles", {})
        if self.key not in tables:
            tables[self.key] = ops.rope_table(meta.pos_ids, freq, self.mult)
        return tables[self.key]


class LatentMixer(Mixer):
    """Latent attention: keys and values are linear maps of a latent of `kv_rank`, beside one rotated key part shared by all
    heads. The cache holds the latent and that part, one row per token. Queries pass a latent of `q_rank`, or none. `sink`: a
    learned score per head joins the softmax; `mask`: a sliding window."""
    kind = "latent_attention"
    extensions = ("ds_mixer_ops", )
    strided = True

    def __init__(self, mx, tp):
        if mx["heads"] % tp:
            raise ValueError(f"{mx['heads']} heads over {tp} ranks")
        self.H, self.d, self.r, self.e = mx["heads"] // tp, mx["dim"], mx["rot_dim"], mx["vdim"]
        self.q_rank, self.kv_rank = int(mx.get("q_rank") or 0), mx["kv_rank"]
        self.scale, self.rot = float(mx["scale"]), Rotation(mx["rot"], mx["rot_dim"])
        self.window = int((mx.get("mask") or {}).get("size") or 0)
        self.sink = bool(mx.get("sink", True))
        self.extra_projections = ("uq_w", ) if self.q_rank else ()
        self.q_cols = self.q_rank or self.H * (self.d + self.r)
        self.rows = self.q_cols + self.kv_rank + self.r
        self.out_width = self.H * self.e

    def parameters(self, device):
        p = {"kv_norm": _f32((self.kv_rank, ), 1.0, device)}
        if self.q_rank:
            p["q_norm"] = _f32((self.q_rank, ), 1.0, device)
        if self.sink:
            p["sink"] = _f32((self.H, ), 0.0, device)
        return p

    def matrices(self, dtype, device):
        m = {"ukv_w": _empty((self.H * (self.d + self.e), self.kv_rank), dtype, device),       # [keys | values]
             "ukt_w": _empty((self.H, self.kv_rank, self.d), dtype, device)}                   # keys, turned over per head
        if self.q_rank:
            m["uq_w"] = _empty((self.H * (self.d + self.r), self.q_rank), dtype, device)
        return m

    def constants(self, device):
        return {"rot_freq": self.rot.frequencies(device)}

    def shard(self, lw, r, tp):
        def s(n, dim=0):
            return _shard(lw[n], r, tp, dim)

        def queries(n):
            w = s(n)
            return self.rot.halves(w.view(self.H, -1, w.shape[1]), self.d).reshape(w.shape)

        uk, dkv = s("uk_w"), lw["dkv_w"]
        dkv = self.rot.halves(dkv[None], self.kv_rank)[0]
        out = {"qkv_w": torch.cat([lw["dq_w"] if self.q_rank else queries("q_w"), dkv]), "ukv_w": torch.cat([uk, s("uv_w")]),
               "ukt_w": uk.view(self.H, self.d, self.kv_rank).transpose(1, 2).contiguous(), "o_w": s("o_w", 1),
               "kv_norm": lw["kv_norm"]}
        if self.q_rank:
            out.update(uq_w=queries("uq_w"), q_norm=lw["q_norm"])
        if self.sink:
            out["sink"] = s("sink")
        return out

    def kv_geometry(self):
        return 1, self.kv_rank + self.r, 0

    def run(self, layer, h, meta, cache, carry):
        proj, lat, Q = layer.project(h, carry), cache.k[layer.layer_idx], self.q_rank
        cq = mixer_ops.latent_prepare(proj if Q else proj[:, self.q_cols:], layer.q_norm if Q else None, layer.kv_norm,
                                      layer.spec.norm_eps, layer.rot_freq, meta, lat, Q, self.rot.mult)
        q = layer._linear(cq, "uq_w") if Q else proj[:, :self.q_cols]
        o = mixer_ops.latent_attention(q.unflatten(1, (self.H, self.d + self.r)), lat, layer.ukv_w, layer.ukt_w, layer.rot_freq,
                                       layer.sink if self.sink else None, meta, self.scale, self.d, self.e, self.window,
                                       self.rot.mult)
        return o.view(h.shape[0], self.out_width)


class WindowAttention(Mixer):
    """Grouped-query attention over a sliding window of `mask.size` keys. Queries and keys are rotated, then divided by their root
    mean square head by head; every head's output is multiplied by the sigmoid of a linear map of the input."""
    kind = "window_attention"
    extensions = ("ds_attn_ops", )
    strided = True

    def __init__(self, mx, tp):
        self.H, self.G, self.dk, self.dv = mx["heads"] // tp, mx["kv_heads"] // tp, mx["dim"], mx["vdim"]
        if mx["heads"] % mx["kv_heads"] or mx["kv_heads"] % tp:
            raise ValueError(f"{mx['heads']} query / {mx['kv_heads']} key heads over {tp} ranks")
        self.scale, self.window = float(mx["scale"]), int((mx.get("mask") or {}).get("size") or 0)
        self.rot = Rotation(mx["rot"], self.dk)
        self.gate = (self.H + self.G) * self.dk + self.G * self.dv   # first of the gates' columns
        self.rows = self.gate + self.H
        self.out_width = self.H * self.dv

    def constants(self, device):
        return {"rot_freq": self.rot.frequencies(device)}

    def shard(self, lw, r, tp):
        def s(n):
            return _shard(lw[n], r, tp)

        def heads(n):   # the kernel turns neighbours
            w = s(n)
            return w if self.rot.neighbours else self._interleave(w)

        return {"qkv_w": torch.cat([heads("q_w"), heads("k_w"), s("v_w"), s("g_w")]), "o_w": _shard(lw["o_w"], r, tp, 1)}

    def _interleave(self, w):
        """Rows (i, i + dims / 2) of every head side by side."""
        half = self.rot.dims // 2
        i = torch.arange(half)
        at = torch.cat([torch.stack([i, i + half], 1).flatten(), torch.arange(2 * half, self.dk)])
        return w.view(-1, self.dk, w.shape[1])[:, at].reshape(w.shape)

    def kv_geometry(self):
        return self.G, self.dk, self.dv

    def run(self, layer, h, meta, cache, carry):
        proj = layer.project(h, carry)
        kc, vc = cache.k[layer.layer_idx], cache.v[layer.layer_idx]
        q = ops.qk_norm_append(proj[:, :self.gate], None, None, layer.spec.norm_eps, None, None, meta.pos_ids, meta.seq_ids,
                               meta.block_tables, kc, vc, self.H, self.rot.angles(layer.rot_freq, meta, carry))
        o = ops.ragged_attention(q, kc, vc, meta, self.scale, window=self.window, gate=proj[:, self.gate:self.gate + self.H])
        return o.reshape(h.shape[0], self.out_width)


class ScanMixer(Mixer):
    """Recurrences S_t = a_t S_(t-1) + b_t k_t v_t^T, o_t = S_t^T q_t + D v_t with a scalar decay per head; the layout of
    the fused projection row tells the kernels where everything is (`mixer_ops.ScanLayout`). Where a tensor-parallel
    split would cut a norm's part, every rank runs all heads and hands its share of the columns on."""
    extensions = ("ds_mixer_ops", "ds_scan_ops")

    def _size(self, layout, parts, tp, split):
        self.lay, self.parts = layout, parts
        self.cols = layout.H * layout.dv
        self.rows = layout.rows
        self.tp_cols = self.cols if split or tp == 1 else self.cols // tp
        if self.cols % self.tp_cols:
            raise ValueError(f"{self.cols} columns over {tp} ranks")
        self.out_width = self.tp_cols

    def parameters(self, device):
        return {"head_norm": _f32((self.cols, ), 1.0, device)}

    def state_geometry(self, dtype):
        la = self.lay
        g = {"state": ((la.H, la.dv, la.dks), torch.float32)}
        if la.taps > 1:
            g["conv"] = ((la.taps - 1, la.channels), dtype)
        return g

    def _share(self, y, layer):
        """Columns of this rank's output projection."""
        if self.tp_cols == self.cols:
            return y
        r = layer.tp_rank * self.tp_cols
        return y[:, r:r + self.tp_cols].contiguous()


class Mamba2Mixer(ScanMixer):
    kind = "mamba2"

    def __init__(self, mx, tp):
        H, G, N, e, parts = mx["heads"], mx["groups"], mx["state"], mx["vdim"], mx["norm_groups"]
        if H % G or (H * e) % parts:
            raise ValueError(f"{H} heads of {e} in {G} groups, normed in {parts} parts")
        self.split = not (H % tp or G % tp or parts % tp)
        if self.split:
            H, G, parts = H // tp, G // tp, parts // tp
        inner = H * e
        self.sections = (inner, inner, G * N, G * N, H)    # z | x | B | C | dt
        self._size(mixer_ops.ScanLayout(rows=sum(self.sections), q=2 * inner + G * N, k=2 * inner, v=inner, gate=0, Hk=G,
                                        H=H, dk=N, dv=e, taps=int(mx["conv"]), conv=inner, channels=inner + 2 * G * N,
                                        dt=2 * inner + 2 * G * N), parts, tp, self.split)

    def parameters(self, device):
        H, C = self.lay.H, self.lay.channels
        return {**super().parameters(device), "conv_w": _f32((C, self.lay.taps), 0.0, device),
                "conv_b": _f32((C, ), 0.0, device), "a_log": _f32((H, ), 0.0, device), "dt_bias": _f32((H, ), 0.0, device),
                "skip": _f32((H, ), 0.0, device)}

    def shard(self, lw, r, tp):
        out = {"qkv_w": lw["in_w"], "conv_w": lw["conv_w"], "conv_b": lw["conv_b"], "a_log": lw["a_log"],
               "dt_bias": lw["dt_bias"], "skip": lw["skip"], "head_norm": lw["head_norm"], "o_w": _shard(lw["o_w"], r, tp, 1)}
        if self.split and tp > 1:
            def cut(t, sections):
                full = [n * tp for n in sections]
                if t.shape[0] != sum(full):
                    raise ValueError(f"{t.shape[0]} rows in the checkpoint, {sum(full)} by the configuration")
                return torch.cat([_shard(p, r, tp) for p in t.split(full)])

            out.update(qkv_w=cut(lw["in_w"], self.sections), conv_w=cut(lw["conv_w"], self.sections[1:4]),
                       conv_b=cut(lw["conv_b"], self.sections[1:4]),
                       **{n: _shard(lw[n], r, tp) for n in ("a_log", "dt_bias", "skip", "head_norm")})
        return out

    def run(self, layer, h, meta, cache, carry):
        proj = layer.project(h, carry)
        st = cache.state[layer.layer_idx]
        y = mixer_ops.decayed_scan(proj, self.lay, st["state"], meta, conv_w=layer.conv_w, conv_b=layer.conv_b,
                                   conv_state=st.get("conv"), a_log=layer.a_log, dt_bias=layer.dt_bias, skip=layer.skip)
        return self._share(mixer_ops.gated_norm(y, proj, self.lay.gate, layer.head_norm, self.parts, layer.spec.norm_eps,
                                                "silu_before"), layer)


class LightningMixer(ScanMixer):
    kind = "lightning"

    def __init__(self, mx, tp):
        H, d, e = mx["heads"], mx["dim"], mx["vdim"]
        if len(mx["decay"]) != H:
            raise ValueError(f"{len(mx['decay'])} decays for {H} heads")
        self.decay = [float(a) for a in mx["decay"]]
        self._size(mixer_ops.ScanLayout(rows=2 * H * (d + e), q=0, k=H * d, v=2 * H * d, gate=2 * H * d + H * e, Hk=H, H=H,
                                        dk=d, dv=e), 1, tp, False)

    def constants(self, device):
        # (a decay of zero: its logarithm as a number whose exponential is zero)
        return {"log_decay": torch.tensor([math.log(a) if a > 0 else -200.0 for a in self.decay], device=device)}

    def shard(self, lw, r, tp):
        return {"qkv_w": torch.cat([lw[n] for n in ("q_w", "k_w", "v_w", "g_w")]), "head_norm": lw["head_norm"],
                "o_w": _shard(lw["o_w"], r, tp, 1)}

    def run(self, layer, h, meta, cache, carry):
        proj = layer.project(h, carry)
        y = mixer_ops.decayed_scan(proj, self.lay, cache.state[layer.layer_idx]["state"], meta, log_decay=layer.log_decay)
        return self._share(mixer_ops.gated_norm(y, proj, self.lay.gate, layer.head_norm, self.parts, layer.spec.norm_eps,
                                                "sigmoid_after"), layer)


class Mamba1Mixer(Mixer):
    """Selective state space: behind a short convolution, every channel carries `state` numbers that decay at rates of their own,
    with step sizes, inputs and read-outs that depend on the token. The steps come through a bottleneck of `dt_rank`. Every
    rank of a tensor-parallel group runs all channels (the bottleneck mixes them) and hands its share on."""
    kind = "mamba1"
    extra_projections = ("x_w", )
    extensions = ("ds_selective_ops", )
    strided = True

    def __init__(self, mx, tp):
        self.inner, self.N, self.R, self.taps = mx["inner"], mx["state"], mx["dt_rank"], int(mx["conv"])
        if self.inner % tp:
            raise ValueError(f"{self.inner} channels over {tp} ranks")
        self.rows, self.out_width = 2 * self.inner, self.inner // tp

    def parameters(self, device):
        C = self.inner
        return {"conv_w": _f32((C, self.taps), 0.0, device), "conv_b": _f32((C, ), 0.0, device),
                "decay": _f32((C, self.N), -1.0, device), "dt_bias": _f32((C, ), 0.0, device), "skip": _f32((C, ), 0.0, device)}

    def matrices(self, dtype, device):
        return {"x_w": _empty((_up8(self.R + 2 * self.N), self.inner), dtype, device),
                "dt_w": _empty((self.inner, self.R), dtype, device)}

    def shard(self, lw, r, tp):
        return {"qkv_w": lw["in_w"], "x_w": _fill_rows(lw["x_w"], self.R + 2 * self.N, "mix.x"), "dt_w": lw["dt_w"],
                "o_w": _shard(lw["o_w"], r, tp, 1), "decay": -lw["a_log"].float().exp(),
                **{n: lw[n] for n in ("conv_w", "conv_b", "dt_bias", "skip")}}

    def state_geometry(self, dtype):
        g = {"state": ((self.inner, -(-self.N // 4) * 4), torch.float32)}
        if self.taps > 1:
            g["conv"] = ((self.taps - 1, self.inner), dtype)
        return g

    def run(self, layer, h, meta, cache, carry):
        proj, st, C = layer.project(h, carry), cache.state[layer.layer_idx], self.inner
        x = mixer_ops.causal_conv(proj[:, :C], layer.conv_w, layer.conv_b, st.get("conv"), meta)
        low = layer._linear(x, "x_w")
        dt = ops.linear(low[:, :self.R], layer.dt_w)
        y = mixer_ops.selective_scan(x, dt, low[:, self.R:self.R + 2 * self.N], proj[:, C:2 * C], layer.dt_bias, layer.decay,
                                     layer.skip, st["state"], proj[:, :C], st.get("conv"), meta)
        if self.out_width == C:
            return y
        r = layer.tp_rank * self.out_width
        return y[:, r:r + self.out_width].contiguous()


class SideMixer(Mixer):
    """A mixer that reads its columns of a fused projection row (from `first` on) and writes its columns of a fused read-out,
    so that several can stand side by side in a layer (`ParallelMixer`). `prefix` names its small weights, `mult` is a factor
    of its output, applied in fp32 ahead of the output projection. Where a tensor-parallel split would cut a norm, every rank
    runs all heads and hands its share of the columns on."""

    def __init__(self, mx, tp, prefix="", first=0, mult=1.0):
        self.prefix, self.first, self.mult = prefix, first, float(mult)

    def _columns(self, cols, tp):
        """`cols`: read-out columns of the heads that run here."""
        self.cols, self.out_width = cols, cols if self.split or tp == 1 else cols // tp
        if cols % self.out_width or (not self.split and cols % tp):
            raise ValueError(f"{cols} columns over {tp} ranks")

    def project(self, lw, r, tp):
        """This rank's rows of the input projection."""
        part = (lambda n: _shard(lw[self.prefix + n], r, tp)) if self.split else (lambda n: lw[self.prefix + n])
        return torch.cat([part(n) for n in self.sections])

    def output(self, lw, r, tp):
        """This rank's columns of the output projection."""
        return _shard(lw[self.prefix + "o_w"], r, tp, 1)

    def small(self, lw, r, tp):
        """The small weights, by name."""
        return {}

    def shard(self, lw, r, tp):
        return {"qkv_w": self.project(lw, r, tp), "o_w": self.output(lw, r, tp), **self.small(lw, r, tp)}

    def weight(self, layer, name):
        return getattr(layer, self.prefix + name)

    def read_out(self, layer, proj, meta, cache, carry, out):
        """Projection rows [T, all columns of the layer] -> out [T, out_width] (columns of a wider matrix)."""
        if self.out_width == self.cols:
            self.heads(layer, proj, meta, cache, carry, out)
            return
        whole = proj.new_empty(proj.shape[0], self.cols)
        self.heads(layer, proj, meta, cache, carry, whole)
        r = layer.tp_rank * self.out_width
        out.copy_(whole[:, r:r + self.out_width])

    def run(self, layer, h, meta, cache, carry):
        proj = layer.project(h, carry)
        out = proj.new_empty(proj.shape[0], self.out_width)
        self.read_out(layer, proj, meta, cache, carry, out)
        return out


class RotaryAttention(SideMixer):
    """Sizes and constants; the weights are the layer's. The output's factor rides on the cached values."""
    kind = "rotary_attention"
    extensions = ("ds_attn_ops", )
    sections = ("q_w", "k_w", "v_w")
    split = False          # the query and key norms run over all heads

    def __init__(self, mx, tp, prefix="", first=0, mult=1.0):
        super().__init__(mx, tp, prefix, first, mult)
        self.H, self.G, self.dk, self.dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
        if self.H % self.G:
            raise ValueError(f"{self.H} query / {self.G} key heads")
        self.scale, self.chunk = float(mx["scale"]), int((mx.get("mask") or {}).get("size") or 0)
        self.rot = Rotation(mx["rot"], self.dk)
        self.rows = (self.H + self.G) * self.dk + self.G * self.dv
        self._columns(self.H * self.dv, tp)

    def parameters(self, device):
        p = self.prefix
        return {p + "bias": _f32((self.rows, ), 0.0, device), p + "q_norm": _f32((self.H * self.dk, ), 1.0, device),
                p + "k_norm": _f32((self.G * self.dk, ), 1.0, device)}

    def constants(self, device):
        # a score of zero without a value in every softmax
        return {self.prefix + "rot_freq": self.rot.frequencies(device), self.prefix + "sink": torch.zeros(self.H, device=device)}

    def small(self, lw, r, tp):
        p = self.prefix
        return {p + "bias": torch.cat([lw[p + n] for n in ("q_b", "k_b", "v_b")]), p + "q_norm": lw[p + "q_norm"],
                p + "k_norm": lw[p + "k_norm"]}

    def kv_geometry(self):
        return self.G, self.dk, self.dv

    def heads(self, layer, proj, meta, cache, carry, out):
        w, kc, vc = self.weight, cache.k[layer.layer_idx], cache.v[layer.layer_idx]
        cs = self.rot.angles(w(layer, "rot_freq"), meta, carry)
        q = ops.qk_rope_append(proj[:, self.first:self.first + self.rows], w(layer, "bias"), w(layer, "q_norm"),
                               w(layer, "k_norm"), layer.spec.norm_eps, cs, meta, kc, vc, self.H, self.mult)
        ops.ragged_attention(q, kc, vc, meta, self.scale, chunk=self.chunk, sink=w(layer, "sink"), out=out)


class HeadScan(SideMixer):
    """A recurrence per head whose read-out is divided by its root mean square head by head: splits by heads."""
    extensions = ("ds_scan_ops", )

    def _heads(self, mx, tp, width):
        """`width`: projection rows per head."""
        H, self.dk, self.dv = mx["heads"], mx["dim"], mx["vdim"]
        self.split = H % tp == 0
        self.H = H // tp if self.split else H
        self.rows = self.H * width
        self._columns(self.H * self.dv, tp)
        a, b = self.first + self.H * self.dk, self.first + 2 * self.H * self.dk
        self.gate = b + self.H * self.dv
        self.at = dict(q=self.first, k=a, v=b, gate=self.gate, Hk=self.H, H=self.H, dk=self.dk, dv=self.dv)

    def state_geometry(self, dtype):
        return {"state": ((self.H, self.dv, -(-self.dk // 8) * 8), torch.float32)}


class MatrixMemory(HeadScan):
    kind = "matrix_memory"
    sections = ("q_w", "k_w", "v_w", "g_w", "i_w", "f_w")

    def __init__(self, mx, tp, prefix="", first=0, mult=1.0):
        super().__init__(mx, tp, prefix, first, mult)
        self.cap = float(mx["gate_cap"])
        self._heads(mx, tp, 2 * mx["dim"] + 2 * mx["vdim"] + 2)

    def parameters(self, device):
        p = self.prefix
        return {p + "i_b": _f32((self.H, ), 0.0, device), p + "f_b": _f32((self.H, ), 0.0, device),
                p + "head_norm": _f32((self.H * self.dv, ), 1.0, device)}

    def small(self, lw, r, tp):
        p = self.prefix
        s = (lambda t: _shard(t, r, tp)) if self.split else (lambda t: t)
        return {p + "i_b": s(lw[p + "i_b"]), p + "f_b": s(lw[p + "f_b"]), p + "head_norm": s(lw[p + "head_norm"]).float() * self.mult}

    def state_geometry(self, dtype):
        dks = -(-self.dk // 8) * 8
        return {**super().state_geometry(dtype), "norm": ((self.H, -(-self.dv // 32), dks), torch.float32),
                "peak": ((self.H, ), torch.float32)}

    def heads(self, layer, proj, meta, cache, carry, out):
        w = self.weight
        y = mixer_ops.matrix_memory(proj, mixer_ops.ScanLayout(rows=proj.shape[1], **self.at), cache.state[layer.layer_idx], meta,
                                    self.gate + self.cols, w(layer, "i_b"), w(layer, "f_b"), self.cap, self.dk**-0.5)
        mixer_ops.gated_norm(y, proj, self.gate, w(layer, "head_norm"), self.H, layer.spec.norm_eps, "sigmoid_after", out)


class Retention(HeadScan):
    kind = "retention"
    sections = ("q_w", "k_w", "v_w", "g_w")

    def __init__(self, mx, tp, prefix="", first=0, mult=1.0):
        super().__init__(mx, tp, prefix, first, mult)
        if mult != 1.0:
            raise NotImplementedError("retention as a scaled side: it has no weight to take the factor")
        if len(mx["decay"]) != mx["heads"]:
            raise ValueError(f"{len(mx['decay'])} decays for {mx['heads']} heads")
        self.decay, self.rot = [float(a) for a in mx["decay"]], Rotation(mx["rot"], mx["dim"])
        self._heads(mx, tp, 2 * mx["dim"] + 2 * mx["vdim"])

    def constants(self, device):
        # (a decay of zero: its logarithm as a number whose exponential is zero)
        return {self.prefix + "log_decay": torch.tensor([math.log(a) if a > 0 else -200.0 for a in self.decay], device=device),
                self.prefix + "rot_freq": self.rot.frequencies(device)}

    def heads(self, layer, proj, meta, cache, carry, out):
        w = self.weight
        ld = w(layer, "log_decay")
        if self.H < len(self.decay):
            ld = ld[layer.tp_rank * self.H:(layer.tp_rank + 1) * self.H]
        y = mixer_ops.retention(proj, mixer_ops.ScanLayout(rows=proj.shape[1], **self.at), cache.state[layer.layer_idx]["state"],
                                meta, ld, self.rot.angles(w(layer, "rot_freq"), meta, carry), self.dk**-0.5)
        mixer_ops.gated_norm(y, proj, self.gate, None, self.H, layer.spec.norm_eps, "silu_after", out)


class ParallelMixer(Mixer):
    """Attention and a matrix memory on the same input: one fused input projection, read-outs side by side, one output
    projection that sums them. At most one side keeps keys and values, at most one a state."""
    kind = "parallel"
    sides = (("left", RotaryAttention), ("right", MatrixMemory))

    def __init__(self, mx, tp):
        self.parts, self.rows, self.out_width = [], 0, 0
        for name, cls in self.sides:
            side = cls(mx[name], tp, name + "_", self.rows, mx[name + "_scale"])
            self.parts.append(side)
            self.rows += side.rows
            self.out_width += side.out_width
        self.extensions = tuple(e for s in self.parts for e in s.extensions)

    def _all(self, f):
        return {k: v for s in self.parts for k, v in f(s).items()}

    def parameters(self, device):
        return self._all(lambda s: s.parameters(device))

    def constants(self, device):
        return self._all(lambda s: s.constants(device))

    def shard(self, lw, r, tp):
        return {"qkv_w": torch.cat([s.project(lw, r, tp) for s in self.parts]),
                "o_w": torch.cat([s.output(lw, r, tp) for s in self.parts], 1), **self._all(lambda s: s.small(lw, r, tp))}

    def kv_geometry(self):
        return next((g for g in (s.kv_geometry() for s in self.parts) if g), None)

    def state_geometry(self, dtype):
        return next((g for g in (s.state_geometry(dtype) for s in self.parts) if g), None)

    def run(self, layer, h, meta, cache, carry):
        proj = layer.project(h, carry)
        out, at = proj.new_empty(proj.shape[0], self.out_width), 0
        for s in self.parts:
            s.read_out(layer, proj, meta, cache, carry, out[:, at:at + s.out_width])
            at += s.out_width
        return out


MIXERS = {m.kind: m for m in (AttentionMixer, LatentMixer, WindowAttention, DeltaMixer, Mamba1Mixer, Mamba2Mixer, LightningMixer,
                              RotaryAttention, MatrixMemory, Retention, ParallelMixer)}


class MLP:
    """What a feed-forward may leave at its default. `rows`: width of the first product's output; `ff`: of the second's input."""
    projections = ("fc1_w", "fc2_w")   # weights that are quantised / re-laid
    entry = "fc1_w"                    # the plain projection of the input, which takes the rows of a residual gate along
    extensions = ()

    def matrices(self, width):
        """Shapes of the weight matrices, by name."""
        return {"fc1_w": (self.rows, width), "fc2_w": (width, self.ff)}

    def operand_order(self, layer):
        """Copies for decoding of weights that are no plain projections."""
        return {}


class ClampedMLP(MLP):
    """Gated feed-forward whose branches are clamped before the product."""
    kind = "dense"
    extensions = ("ds_hybrid_ops", )

    def __init__(self, ml, tp):
        if ml["ff"] % tp:
            raise ValueError(f"feed-forward width {ml['ff']} over {tp} ranks")
        self.ff, self.limit = ml["ff"] // tp, float(ml["limit"])
        self.rows = 2 * self.ff

    def shard(self, lw, r, tp):
        return {"fc1_w": torch.cat([_shard(lw["gate_w"], r, tp), _shard(lw["up_w"], r, tp)]),
                "fc2_w": _shard(lw["down_w"], r, tp, 1)}

    def run(self, layer, h, carry):
        if "fc1_w" in layer.quant or layer.gated:
            mid = ops.clamped_glu(layer.project(h, carry, self).contiguous(), self.limit)
        else:
            mid = ops.glu_linear(h, layer.fc1_w, layer.sh.get("fc1_w"), self.limit)
        return layer._linear(mid, "fc2_w")


class GatedMLP(MLP):
    """Gated feed-forward: down (silu(gate x) * up x)."""
    kind = "silu_glu"
    extensions = ("ds_expert_ops", )

    def __init__(self, ml, tp):
        if ml["ff"] % tp:
            raise ValueError(f"feed-forward width {ml['ff']} over {tp} ranks")
        self.ff = ml["ff"] // tp
        self.rows = 2 * self.ff

    def shard(self, lw, r, tp):
        return {"fc1_w": torch.cat([_shard(lw["gate_w"], r, tp), _shard(lw["up_w"], r, tp)]),
                "fc2_w": _shard(lw["down_w"], r, tp, 1)}

    def run(self, layer, h, carry):
        return layer._linear(expert_ops.row_act(layer.project(h, carry, self), "silu_glu"), "fc2_w")


class GeluMLP(MLP):
    """Feed-forward without a gate: down gelu(up x), the gelu of the error function."""
    kind = "gelu"
    extensions = ("ds_mixer_ops", )

    def __init__(self, ml, tp):
        if ml["ff"] % tp:
            raise ValueError(f"feed-forward width {ml['ff']} over {tp} ranks")
        self.ff = self.rows = ml["ff"] // tp

    def shard(self, lw, r, tp):
        return {"fc1_w": _shard(lw["up_w"], r, tp), "fc2_w": _shard(lw["down_w"], r, tp, 1)}

    def run(self, layer, h, carry):
        if "fc1_w" in layer.quant or layer.gated:
            mid = mixer_ops.gelu(layer.project(h, carry, self).contiguous())
        else:
            mid = ops.linear(h, layer.fc1_w, layer.sh.get("fc1_w"), act="gelu")
        return layer._linear(mid, "fc2_w")


class RoutedMLP(MLP):
    """Mixture of experts: gated (silu) ones, or plain ones with `act` between their two maps. The experts form equal groups; those
    of the best groups (by their `best` best members) compete, the best are weighted by their scores (the softmax over all, or
    sigmoids), divided by the scores' sum, times a scale. `shared`: an expert that every token takes. Every rank routes for
    itself and holds a slice of every expert."""
    kind = "routed"
    extensions = ("ds_expert_ops", )
    entry = "shared1_w"

    def __init__(self, ml, tp):
        ro = ml["router"]
        groups = ro.get("groups") or {}
        self.E, self.top = int(ro["experts"]), int(ro["top"])
        self.groups, self.keep = int(groups.get("count", 1)), int(groups.get("keep", 1))
        self.act, self.shared = ml.get("act", "silu_glu"), int((ml.get("shared") or {}).get("ff") or 0)
        self.how = dict(score=ro.get("score", "softmax"), best=int(groups.get("best", 1)), scale=float(ro.get("scale", 1.0)),
                        act=self.act)
        if ml["expert"]["ff"] % tp or self.shared % tp:
            raise ValueError(f"expert widths {ml['expert']['ff']}, {self.shared} over {tp} ranks")
        if self.groups < 1 or self.E % self.groups or not 1 <= self.keep <= self.groups or \
                not 1 <= self.top <= self.keep * (self.E // self.groups):
            raise ValueError(f"{self.top} of {self.E} experts, {self.keep} of {self.groups} groups")
        self.ff, self.shared, self.parts = ml["expert"]["ff"] // tp, self.shared // tp, 2 if self.act == "silu_glu" else 1
        self.rows = self.parts * self.shared
        self.projections = ("shared1_w", "shared2_w") if self.shared else ()

    def matrices(self, width):
        m = {"router_w": (self.E, width), "fc1_w": (self.E, self.parts * self.ff, width), "fc2_w": (self.E, width, self.ff)}
        if self.shared:
            m.update(shared1_w=(self.rows, width), shared2_w=(width, self.shared))
        return m

    def shard(self, lw, r, tp):
        names = ("gate", "up")[2 - self.parts:]
        out = {"router_w": lw["router_w"], "fc1_w": torch.cat([_shard(lw[f"experts_{n}"], r, tp, 1) for n in names], 1),
               "fc2_w": _shard(lw["experts_down"], r, tp, 2)}
        if self.shared:
            out.update(shared1_w=torch.cat([_shard(lw[f"shared_{n}"], r, tp) for n in names]),
                       shared2_w=_shard(lw["shared_down"], r, tp, 1))
        return out

    def operand_order(self, layer):
        """The expert weights once more as the products read them best, by name (nothing where the sizes forbid it)."""
        if self.ff % 32:   # (gate and up rows are tiled on their own)
            return {}
        both = expert_ops.operand_order(layer.fc1_w.data), expert_ops.operand_order(layer.fc2_w.data)
        return {} if any(w is None for w in both) else {"experts": both}

    def run(self, layer, h, carry):
        first = layer.project(h, carry, self) if self.shared or layer.gated else None
        y = expert_ops.experts(h, layer.router_w, layer.fc1_w, layer.fc2_w, self.top, self.groups, self.keep,
                               layer.sh.get("experts"), **self.how)
        if self.shared:
            y.base = layer._linear(expert_ops.row_act(first, self.act), "shared2_w")
        return y if layer.tp == 1 else y.sum()   # ranks exchange plain sums


MLPS = {m.kind: m for m in (ClampedMLP, GatedMLP, GeluMLP, RoutedMLP)}


class TokenSide:
    """Per-layer token input: proj(gelu(gate x) * e), e the layer's part of a side embedding of the token."""
    extensions = ("ds_mixer_ops", )

    def __init__(self, dim, layer_idx):
        self.dim, self.first = dim, layer_idx * dim

    def shard(self, lw):
        return {"side_gate_w": lw["side_gate_w"], "side_proj_w": lw["side_proj_w"]}

    def run(self, layer, h, carry):
        g = mixer_ops.token_gate(layer._linear(h, "side_gate_w"), carry["ids"], carry["side_embed"], self.first)
        return layer._linear(g, "side_proj_w")


class DSHybridLayer(ProjectionLayer):
    """One layer of a hybrid decoder: the residual around a mixer and, where the spec has them, a feed-forward and a
    token-side input."""

    def __init__(self, spec, layer_idx, tp_group=None, tp_size=1, dtype=torch.bfloat16, device=None):
        super().__init__(spec, layer_idx, tp_group, tp_size)
        ls, W = spec.layer_specs[layer_idx], spec.hidden_size
        if ls["type"] not in MIXERS:
            raise NotImplementedError(f"layer {layer_idx}: no mixer {ls['type']!r}")
        residual = RESIDUALS[spec.residual]
        self.tp_rank, self.gated = 0, spec.residual_gate
        self.mixer = MIXERS[ls["type"]](ls["mixer"], tp_size)
        self.res1 = residual(spec, device)
        self.qkv_w = _empty((self._rows(self.mixer.rows), W), dtype, device)
        self.o_w = _empty((W, self.mixer.out_width), dtype, device)
        for name, p in {**self.mixer.parameters(device), **self.mixer.matrices(dtype, device)}.items():
            self.register_parameter(name, p)
        for name, t in self.mixer.constants(device).items():
            self.register_buffer(name, t, persistent=False)
        self.mlp = self.side = None
        if ls.get("mlp"):
            kind = ls["mlp"].get("kind")
            if kind not in MLPS:
                raise NotImplementedError(f"layer {layer_idx}: no feed-forward {kind!r}")
            self.mlp = MLPS[kind](ls["mlp"], tp_size)
            self.res2 = residual(spec, device)
            shapes = self.mlp.matrices(W)
            if self.gated:
                shapes[self.mlp.entry] = (self._rows(self.mlp.rows), W)
            for name, shape in shapes.items():
                self.register_parameter(name, _empty(shape, dtype, device))
        if spec.token_side:
            self.side = TokenSide(spec.token_side, layer_idx)
            self.res_side = residual(spec, device, side=True)
            self.side_gate_w = _empty((spec.token_side, W), dtype, device)
            self.side_proj_w = _empty((W, spec.token_side), dtype, device)

    def projection_names(self):
        return ("qkv_w", "o_w") + self.mixer.extra_projections + (self.mlp.projections if self.mlp else ()) + \
            (("side_gate_w", "side_proj_w") if self.side else ())

    def _rows(self, own):
        """Rows of a sublayer's first projection: its own and, behind a whole number of 16-byte pieces, the residual gate's."""
        return _up8(own) + self.spec.hidden_size if self.gated else own

    def _linear(self, x, name, bias=None):
        if name in self.quant:
            return super()._linear(x, name, bias)
        return ops.linear(x, getattr(self, name), self.sh.get(name))

    def project(self, h, carry, mlp=None):
        """The input projection of the mixer (or the feed-forward). What the residual gate's rows make of h goes to
        carry["gate"]."""
        part = mlp or self.mixer
        y = self._linear(h, mlp.entry if mlp else "qkv_w")
        if not self.gated:
            return y
        carry["gate"] = y[:, _up8(part.rows):]
        own = y[:, :part.rows]
        return own if mlp or part.strided else own.contiguous()

    def add_decode_layout(self):
        """Shuffled copies of the projections whose shape allows one (see the base class)."""
        from ...ops.bf16_gemv import Bf16Weight
        if self.quant:
            return False
        self.sh = {n: Bf16Weight(w.data) for n, w in ((n, getattr(self, n)) for n in self.projection_names())
                   if w.is_cuda and Bf16Weight.supported(w.data)}
        if self.mlp:
            self.sh.update(self.mlp.operand_order(self))
        return bool(self.sh)

    def shard(self, lw, r, tp):
        """Canonical full weights -> {attribute path: this rank's tensor}."""
        out = self.mixer.shard(lw, r, tp)
        if self.mlp:
            out.update(self.mlp.shard(lw, r, tp))
        if self.side:
            out.update(self.side.shard(lw))
            out["res_side.post_w" if hasattr(self.res_side, "post_w") else "res_side.norm_w"] = lw["side_norm_w"]
        for q in (1, 2) if self.mlp else (1, ):
            out[f"res{q}.norm_w"] = lw[f"norm{q}_w"]
            for n in ("in", "out", "mix"):
                if f"hc{q}_{n}" in lw:
                    out[f"res{q}.{'in_' if n == 'in' else n}"] = lw[f"hc{q}_{n}"]
            if f"post{q}_w" in lw:
                out[f"res{q}.post_w"] = lw[f"post{q}_w"]
            if self.gated:
                name, part, gate = "qkv_w" if q == 1 else self.mlp.entry, self.mixer if q == 1 else self.mlp, lw[f"rg{q}_w"]
                own = out.get(name, gate.new_empty(0, gate.shape[1]))
                out[name] = torch.cat([_fill_rows(own, part.rows, name), gate])
                out[f"res{q}.gate_b"] = lw[f"rg{q}_b"]
        return out

    def forward(self, x, pending, meta, cache, carry):
        """x: the residual, fp32. `pending`: (output, residual weights, gate) of the sublayer before, not yet added, or the
        input of the first layer. Returns this layer's last sublayer as pending."""
        h = pending if torch.is_tensor(pending) else self.res1.enter(self.spec, x, pending)
        y = self._allreduce(self._linear(self.mixer.run(self, h, meta, cache, carry), "o_w"))
        pending = (y, self.res1, carry.pop("gate", None))
        if self.mlp:
            h = self.res2.enter(self.spec, x, pending)
            y = self._allreduce(self.mlp.run(self, h, carry))
            pending = (y, self.res2, carry.pop("gate", None))
        if self.side:
            h = self.res_side.enter(self.spec, x, pending)
            pending = (self.side.run(self, h, carry), self.res_side, None)
        return pending


class DSHybridModel(DSInferenceModel):
    layer_class = DSHybridLayer

    def __init__(self, spec, tp_group=None, tp_size=1, tp_rank=0, dtype=torch.bfloat16, device=None):
        super().__init__(spec, tp_group, tp_size, tp_rank, dtype, device)
        if torch.device(device or "cpu").type == "cuda":  # all at once: in a fresh checkout they compile side by side
            parts = [p for la in self.layers for p in (la.mixer, la.mlp, la.side, la.res1) if p]
            op_builder.prepare(sorted({"ds_gemv_ops", *(e for p in parts for e in p.extensions)}))
        self.norm_w = _f32((spec.hidden_size, ), 1.0, device)  # norms read the fp32 residual
        if spec.token_side:
            self.side_embed = _empty((spec.vocab_size, spec.token_side * spec.num_layers), dtype, device)
        for layer in self.layers:
            layer.tp_rank = tp_rank

    # ------------------------------------------------------------------------------------------ cache
    def kv_geometry(self):
        return [la.mixer.kv_geometry() for la in self.layers]

    def state_geometry(self):
        return [la.mixer.state_geometry(self.dtype) for la in self.layers]

    def shard_layer(self, idx, lw):
        return self.layers[idx].shard(lw, self.tp_rank, self.tp_size)

    def shard_top(self, top):
        """Tensors beside the layers' that only this kind of model has -> {attribute: tensor}."""
        return {"side_embed": top["side_embed"]} if self.spec.token_side else {}

    # ------------------------------------------------------------------------------------------ forward
    def forward(self, input_ids, meta, all_logits=False):
        raise NotImplementedError("hybrid decoders are served by the ragged engine (inference v2)")

    @torch.no_grad()
    def forward_ragged(self, tokens, meta, trace=None):
        """tokens [T] -> logits of rows `meta.last_idx`. `trace` (a list) receives the residual (the sum of its streams)
        after every layer (a debugging aid: it costs a pass per layer)."""
        spec, ids = self.spec, tokens.to(torch.int32)
        x, pending = RESIDUALS[spec.residual].begin(self, ids)
        carry = {"ids": ids, "side_embed": getattr(self, "side_embed", None)}
        for layer in self.layers:
            pending = layer(x, pending, meta, self.cache, carry)
            if trace is not None:
                y, r, gate = pending
                trace.append(r.peek(spec, x, y, gate))
        if meta.last_idx.numel() == 0:
            return tokens.new_empty((0, spec.vocab_size), dtype=self.dtype)
        y, r, gate = pending
        return self._logits(r.finish(self, x, y, meta.last_idx.to(torch.int32), gate))

    def _logits(self, h):
        return self._gather_vocab(ops.linear(h, self.lm_head, getattr(self, "lm_head_sh", None)))


def model_class(spec):
    """The model class a spec describes."""
    return DSHybridModel if spec.layer_specs else DSInferenceModel
