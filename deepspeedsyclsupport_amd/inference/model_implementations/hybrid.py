"""Decoders whose layers differ from one another: every layer names its mixer (attention or a recurrence), the
mixer's sizes and its feed-forward (`DSModelSpec.layer_specs`), and the residual may run in several streams.

`DSHybridModel` is a `DSInferenceModel`: the engines, the ragged batch, the paged cache, sampling, quantisation and
serialisation treat it like any other. What is different sits in one class per mechanism, each with its sizes and
constants as parameters:

* `StreamResidual`  S fp32 residual streams, mixed by small matrices around every sublayer, fused with the pre-norm
* `AttentionMixer`  GQA, key and value widths of their own, per-head query / key RMS norm, score cap, chunked
                    visibility, value mixing with an earlier layer; K / V live in the blocked cache
* `DeltaMixer`      gated delta rule behind short convolutions; its fp32 state lives in a slot per sequence
* `ClampedMLP`      gated feed-forward with clamped gate and up branches

Per sublayer the launches are: residual + norm, one fused input projection, the mixer's kernels, the output projection.
"""
import torch
import torch.nn as nn

from ...ops import hybrid_ops as ops
from .transformer import DSInferenceModel, ProjectionLayer


def _f32(shape, fill, device):
    return nn.Parameter(torch.full(shape, fill, dtype=torch.float32, device=device), requires_grad=False)


def _empty(shape, dtype, device):
    return nn.Parameter(torch.empty(*shape, dtype=dtype, device=device), requires_grad=False)


def _shard(t, r, tp, dim=0):
    return t if tp == 1 else t.chunk(tp, dim)[r]


class StreamResidual(nn.Module):
    """Mixing weights of one sublayer: in_ [S], mix [S from, S to], out [S] (identity for a plain residual)."""

    def __init__(self, streams, width, device):
        super().__init__()
        self.norm_w = _f32((width, ), 1.0, device)
        self.in_ = _f32((streams, ), 1.0, device)
        self.out = _f32((streams, ), 1.0, device)
        self.mix = _f32((streams, streams), 1.0, device)


class AttentionMixer:
    """Sizes and constants of an attention mixer; the weights are the layer's."""
    kind = "attention"

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

    def run(self, layer, h, meta, cache, carry):
        qkv = layer._linear(h, "qkv_w")
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


class DeltaMixer:
    """Sizes of a gated-delta-rule mixer; the weights are the layer's."""
    kind = "delta"

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

    def run(self, layer, h, meta, cache, carry):
        proj = layer._linear(h, "qkv_w")
        st = cache.state[layer.layer_idx]
        return ops.delta_rule(proj, layer.conv_w, layer.a_log, layer.dt_bias, layer.head_norm, layer.spec.norm_eps,
                              st["state"], st["conv"], meta, self.Hk, self.H, self.dk, self.dv)


MIXERS = {m.kind: m for m in (AttentionMixer, DeltaMixer)}


class ClampedMLP:
    """Gated feed-forward whose branches are clamped before the product."""
    kind = "dense"

    def __init__(self, ml, tp):
        if ml["ff"] % tp:
            raise ValueError(f"feed-forward width {ml['ff']} over {tp} ranks")
        self.ff, self.limit = ml["ff"] // tp, float(ml["limit"])

    def shard(self, lw, r, tp):
        return {"fc1_w": torch.cat([_shard(lw["gate_w"], r, tp), _shard(lw["up_w"], r, tp)]),
                "fc2_w": _shard(lw["down_w"], r, tp, 1)}

    def run(self, layer, h):
        if "fc1_w" in layer.quant:
            mid = ops.clamped_glu(layer._linear(h, "fc1_w"), self.limit)
        else:
            mid = ops.glu_linear(h, layer.fc1_w, layer.sh.get("fc1_w"), self.limit)
        return layer._linear(mid, "fc2_w")


MLPS = {m.kind: m for m in (ClampedMLP, )}


class DSHybridLayer(ProjectionLayer):
    """One layer of a hybrid decoder: residual streams around a mixer and, unless the spec says none, a feed-forward."""

    def __init__(self, spec, layer_idx, tp_group=None, tp_size=1, dtype=torch.bfloat16, device=None):
        super().__init__(spec, layer_idx, tp_group, tp_size)
        ls, W = spec.layer_specs[layer_idx], spec.hidden_size
        if ls["type"] not in MIXERS:
            raise NotImplementedError(f"layer {layer_idx}: no mixer {ls['type']!r}")
        self.mixer = MIXERS[ls["type"]](ls["mixer"], tp_size)
        self.res1 = StreamResidual(spec.streams, W, device)
        self.qkv_w = _empty((self.mixer.rows, W), dtype, device)
        self.o_w = _empty((W, self.mixer.out_width), dtype, device)
        for name, p in self.mixer.parameters(device).items():
            self.register_parameter(name, p)
        self.mlp = None
        if ls.get("mlp"):
            kind = ls["mlp"].get("kind")
            if kind not in MLPS:
                raise NotImplementedError(f"layer {layer_idx}: no feed-forward {kind!r}")
            self.mlp = MLPS[kind](ls["mlp"], tp_size)
            self.res2 = StreamResidual(spec.streams, W, device)
            self.fc1_w = _empty((2 * self.mlp.ff, W), dtype, device)
            self.fc2_w = _empty((W, self.mlp.ff), dtype, device)

    def projection_names(self):
        return ("qkv_w", "o_w") + (("fc1_w", "fc2_w") if self.mlp else ())

    def _linear(self, x, name, bias=None):
        if name in self.quant:
            return super()._linear(x, name, bias)
        return ops.linear(x, getattr(self, name), self.sh.get(name))

    def add_decode_layout(self):
        """Shuffled copies of the projections whose shape allows one (see the base class)."""
        from ...ops.bf16_gemv import Bf16Weight
        if self.quant:
            return False
        self.sh = {n: Bf16Weight(w.data) for n, w in ((n, getattr(self, n)) for n in self.projection_names())
                   if w.is_cuda and Bf16Weight.supported(w.data)}
        return bool(self.sh)

    def shard(self, lw, r, tp):
        """Canonical full weights -> {attribute path: this rank's tensor}."""
        out = self.mixer.shard(lw, r, tp)
        if self.mlp:
            out.update(self.mlp.shard(lw, r, tp))
        for q in (1, 2) if self.mlp else (1, ):
            out[f"res{q}.norm_w"] = lw[f"norm{q}_w"]
            for n in ("in", "out", "mix"):
                if f"hc{q}_{n}" in lw:
                    out[f"res{q}.{'in_' if n == 'in' else n}"] = lw[f"hc{q}_{n}"]
        return out

    def _enter(self, x, pending, res):
        """Close the previous sublayer (its output and residual weights) and norm this one's input."""
        y, prev = pending
        return ops.stream_norm(x, y, prev.mix, prev.out, self.spec.residual_mult, res.in_, res.norm_w,
                               self.spec.norm_eps)

    def forward(self, x, pending, meta, cache, carry):
        """x [T, S, W] streams. `pending`: (output, residual weights) of the sublayer before, not yet added, or the
        already normed input of the first layer. Returns this layer's last sublayer as pending."""
        h = pending if torch.is_tensor(pending) else self._enter(x, pending, self.res1)
        y = self._allreduce(self._linear(self.mixer.run(self, h, meta, cache, carry), "o_w"))
        pending = (y, self.res1)
        if self.mlp:
            h = self._enter(x, pending, self.res2)
            pending = (self._allreduce(self.mlp.run(self, h)), self.res2)
        return pending


class DSHybridModel(DSInferenceModel):
    layer_class = DSHybridLayer

    def __init__(self, spec, tp_group=None, tp_size=1, tp_rank=0, dtype=torch.bfloat16, device=None):
        super().__init__(spec, tp_group, tp_size, tp_rank, dtype, device)
        self.norm_w = _f32((spec.hidden_size, ), 1.0, device)  # norms read the fp32 streams

    # ------------------------------------------------------------------------------------------ cache
    def kv_geometry(self):
        return [(m.G, m.dk, m.dv) if m.kind == "attention" else None for m in (la.mixer for la in self.layers)]

    def state_geometry(self):
        return [{"state": ((m.H, m.dv, -(-m.dk // 4) * 4), torch.float32), "conv": ((m.taps - 1, m.channels), self.dtype)}
                if m.kind == "delta" else None for m in (la.mixer for la in self.layers)]

    def shard_layer(self, idx, lw):
        return self.layers[idx].shard(lw, self.tp_rank, self.tp_size)

    # ------------------------------------------------------------------------------------------ forward
    def forward(self, input_ids, meta, all_logits=False):
        raise NotImplementedError("hybrid decoders are served by the ragged engine (inference v2)")

    @torch.no_grad()
    def forward_ragged(self, tokens, meta, trace=None):
        """tokens [T] -> logits of rows `meta.last_idx`. `trace` (a list) receives the sum of the streams after every
        layer (a debugging aid: it costs a pass per layer)."""
        spec = self.spec
        x = torch.empty(tokens.numel(), spec.streams, spec.hidden_size, dtype=torch.float32, device=self.embed.device)
        first = self.layers[0].res1
        pending = ops.stream_norm(x, None, None, None, 1.0, first.in_, first.norm_w, spec.norm_eps,
                                  ids=tokens.to(torch.int32), embed=self.embed)
        carry = {}
        for layer in self.layers:
            pending = layer(x, pending, meta, self.cache, carry)
            if trace is not None:
                y, r = pending
                trace.append((torch.einsum("st,nsw->ntw", r.mix, x) +
                              spec.residual_mult * r.out[None, :, None] * y[:, None].float()).sum(1))
        if meta.last_idx.numel() == 0:
            return tokens.new_empty((0, spec.vocab_size), dtype=self.dtype)
        y, r = pending
        h = ops.stream_norm(x, y, r.mix, r.out, spec.residual_mult, None, self.norm_w, spec.norm_eps,
                            rows=meta.last_idx.to(torch.int32))
        return self._logits(h)

    def _logits(self, h):
        return self._gather_vocab(ops.linear(h, self.lm_head, getattr(self, "lm_head_sh", None)))


def model_class(spec):
    """The model class a spec describes."""
    return DSHybridModel if spec.layer_specs else DSInferenceModel
