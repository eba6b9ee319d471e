"""Decoders whose layers differ from one another: every layer names its mixer (attention or a recurrence), the
mixer's sizes and its feed-forward (`DSModelSpec.layer_specs`), and the residual may run in several streams.

`DSHybridModel` is a `DSInferenceModel`: the engines, the ragged batch, the paged cache, sampling, quantisation and
serialisation treat it like any other. What is different sits in one class per mechanism, each with its sizes and
constants as parameters:

* `StreamResidual`    S fp32 residual streams, mixed by small matrices around every sublayer, fused with the pre-norm
* `PostNormResidual`  one fp32 residual; the sublayers read it as it is and their outputs are RMS-normed before the sum
* `AttentionMixer`    GQA, key and value widths of their own, per-head query / key RMS norm, score cap, chunked
                      visibility, value mixing with an earlier layer; K / V live in the blocked cache
* `LatentMixer`       attention over a shared low-rank latent with a rotated key part and a softmax sink; only the latent
                      and that key part are cached
* `DeltaMixer`        gated delta rule behind short convolutions; its fp32 state lives in a slot per sequence
* `Mamba2Mixer`       state-space recurrence with a scalar decay per head and token behind a short convolution
* `LightningMixer`    linear attention with a constant decay per head
* `ClampedMLP`        gated feed-forward with clamped gate and up branches
* `GeluMLP`           plain feed-forward with the exact gelu
* `TokenSide`         a small embedding per layer and token, gated by the residual

Per sublayer the launches are: residual + norm, one fused input projection, the mixer's kernels, the output projection.
"""
import math

import torch
import torch.nn as nn

from ...ops import hybrid_ops as ops
from ...ops import mixer_ops
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

    @staticmethod
    def begin(model, ids):
        """Residual of a batch and the first sublayer's input."""
        spec, first = model.spec, model.layers[0].res1
        x = torch.empty(ids.numel(), spec.streams, spec.hidden_size, dtype=torch.float32, device=model.embed.device)
        return x, ops.stream_norm(x, None, None, None, 1.0, first.in_, first.norm_w, spec.norm_eps, ids=ids,
                                  embed=model.embed)

    def enter(self, spec, x, pending):
        """Close the sublayer before (its output and residual weights) and norm this one's input."""
        y, prev = pending
        return ops.stream_norm(x, y, prev.mix, prev.out, spec.residual_mult, self.in_, self.norm_w, spec.norm_eps)

    def finish(self, model, x, y, rows):
        """Normed output rows of the model; this is the last sublayer's residual."""
        return ops.stream_norm(x, y, self.mix, self.out, model.spec.residual_mult, None, model.norm_w,
                               model.spec.norm_eps, rows=rows)

    def peek(self, spec, x, y):
        """Sum of the streams after this sublayer."""
        return (torch.einsum("st,nsw->ntw", self.mix, x) +
                spec.residual_mult * self.out[None, :, None] * y[:, None].float()).sum(1)


class PostNormResidual(nn.Module):
    """Norm weight of one sublayer's output: x <- x + y / rms(y) * w."""

    def __init__(self, streams, width, device):
        super().__init__()
        self.norm_w = _f32((width, ), 1.0, device)

    @staticmethod
    def begin(model, ids):
        x = torch.empty(ids.numel(), model.spec.hidden_size, dtype=torch.float32, device=model.embed.device)
        return x, mixer_ops.post_norm(x, None, None, 0.0, ids=ids, embed=model.embed)

    def enter(self, spec, x, pending):
        y, prev = pending
        return mixer_ops.post_norm(x, y, prev.norm_w, spec.norm_eps)

    def finish(self, model, x, y, rows):
        return mixer_ops.post_norm(x, y, self.norm_w, model.spec.norm_eps, rows=rows, final_w=model.norm_w,
                                   mult=model.spec.logit_scale)

    def peek(self, spec, x, y):
        y = y.float()
        return x + y * torch.rsqrt(y.pow(2).mean(-1, keepdim=True) + spec.norm_eps) * self.norm_w


RESIDUALS = {"streams": StreamResidual, "post_norm": PostNormResidual}


class Mixer:
    """What a mixer may leave at its default. `rows`: width of the fused input projection; `out_width`: of its output."""
    extra_projections = ()   # names of weight matrices beside the input and output projection

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


class DeltaMixer(Mixer):
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

    def state_geometry(self, dtype):
        return {"state": ((self.H, self.dv, -(-self.dk // 4) * 4), torch.float32), "conv": ((self.taps - 1, self.channels),
                                                                                         dtype)}

    def run(self, layer, h, meta, cache, carry):
        proj = layer._linear(h, "qkv_w")
        st = cache.state[layer.layer_idx]
        return ops.delta_rule(proj, layer.conv_w, layer.a_log, layer.dt_bias, layer.head_norm, layer.spec.norm_eps,
                              st["state"], st["conv"], meta, self.Hk, self.H, self.dk, self.dv)


class LatentMixer(Mixer):
    """Latent attention: queries through a latent of `q_rank`; keys and values are linear maps of a latent of `kv_rank`,
    beside one rotated key part shared by all heads. The cache holds the latent and that part, one row per token."""
    kind = "latent_attention"
    extra_projections = ("uq_w", )

    def __init__(self, mx, tp):
        if mx["heads"] % tp:
            raise ValueError(f"{mx['heads']} heads over {tp} ranks")
        self.H, self.d, self.r, self.e = mx["heads"] // tp, mx["dim"], mx["rot_dim"], mx["vdim"]
        self.q_rank, self.kv_rank = mx["q_rank"], mx["kv_rank"]
        self.scale, self.base, self.rot = float(mx["scale"]), float(mx["rot"]["base"]), int(mx["rot"]["dims"])
        if self.rot % 2 or self.rot > self.r:
            raise ValueError(f"{self.rot} rotated of {self.r} dimensions")
        self.rows = self.q_rank + self.kv_rank + self.r
        self.out_width = self.H * self.e

    def parameters(self, device):
        return {"q_norm": _f32((self.q_rank, ), 1.0, device), "kv_norm": _f32((self.kv_rank, ), 1.0, device),
                "sink": _f32((self.H, ), 0.0, device)}

    def matrices(self, dtype, device):
        return {"uq_w": _empty((self.H * (self.d + self.r), self.q_rank), dtype, device),
                "ukv_w": _empty((self.H * (self.d + self.e), self.kv_rank), dtype, device),    # [keys | values]
                "ukt_w": _empty((self.H, self.kv_rank, self.d), dtype, device)}                # keys, turned over per head

    def constants(self, device):
        i = torch.arange(self.rot // 2, dtype=torch.float64)
        return {"rot_freq": (self.base**(-2 * i / max(self.rot, 1))).to(device)}

    def shard(self, lw, r, tp):
        def s(n, dim=0):
            return _shard(lw[n], r, tp, dim)

        uk = s("uk_w")
        return {"qkv_w": torch.cat([lw["dq_w"], lw["dkv_w"]]), "uq_w": s("uq_w"), "ukv_w": torch.cat([uk, s("uv_w")]),
                "ukt_w": uk.view(self.H, self.d, self.kv_rank).transpose(1, 2).contiguous(), "o_w": s("o_w", 1),
                "q_norm": lw["q_norm"], "kv_norm": lw["kv_norm"], "sink": s("sink")}

    def kv_geometry(self):
        return 1, self.kv_rank + self.r, 0

    def run(self, layer, h, meta, cache, carry):
        down = layer._linear(h, "qkv_w")
        lat = cache.k[layer.layer_idx]
        cq = mixer_ops.latent_prepare(down, layer.q_norm, layer.kv_norm, layer.spec.norm_eps, layer.rot_freq, meta, lat,
                                      self.q_rank)
        q = layer._linear(cq, "uq_w").view(-1, self.H, self.d + self.r)
        o = mixer_ops.latent_attention(q, lat, layer.ukv_w, layer.ukt_w, layer.rot_freq, layer.sink, meta, self.scale,
                                       self.d, self.e)
        return o.view(h.shape[0], self.out_width)


class ScanMixer(Mixer):
    """Recurrences S_t = a_t S_(t-1) + b_t k_t v_t^T, o_t = S_t^T q_t + D v_t with a scalar decay per head; the layout of
    the fused projection row tells the kernels where everything is (`mixer_ops.ScanLayout`). Where a tensor-parallel
    split would cut a norm's part, every rank runs all heads and hands its share of the columns on."""

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
        proj = layer._linear(h, "qkv_w")
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
        proj = layer._linear(h, "qkv_w")
        y = mixer_ops.decayed_scan(proj, self.lay, cache.state[layer.layer_idx]["state"], meta, log_decay=layer.log_decay)
        return self._share(mixer_ops.gated_norm(y, proj, self.lay.gate, layer.head_norm, self.parts, layer.spec.norm_eps,
                                                "sigmoid_after"), layer)


MIXERS = {m.kind: m for m in (AttentionMixer, LatentMixer, DeltaMixer, Mamba2Mixer, LightningMixer)}


class ClampedMLP:
    """Gated feed-forward whose branches are clamped before the product."""
    kind = "dense"

    def __init__(self, ml, tp):
        if ml["ff"] % tp:
            raise ValueError(f"feed-forward width {ml['ff']} over {tp} ranks")
        self.ff, self.limit = ml["ff"] // tp, float(ml["limit"])
        self.rows = 2 * self.ff

    def shard(self, lw, r, tp):
        return {"fc1_w": torch.cat([_shard(lw["gate_w"], r, tp), _shard(lw["up_w"], r, tp)]),
                "fc2_w": _shard(lw["down_w"], r, tp, 1)}

    def run(self, layer, h):
        if "fc1_w" in layer.quant:
            mid = ops.clamped_glu(layer._linear(h, "fc1_w"), self.limit)
        else:
            mid = ops.glu_linear(h, layer.fc1_w, layer.sh.get("fc1_w"), self.limit)
        return layer._linear(mid, "fc2_w")


class GeluMLP:
    """Feed-forward without a gate: down gelu(up x), the gelu of the error function."""
    kind = "gelu"

    def __init__(self, ml, tp):
        if ml["ff"] % tp:
            raise ValueError(f"feed-forward width {ml['ff']} over {tp} ranks")
        self.ff = self.rows = ml["ff"] // tp

    def shard(self, lw, r, tp):
        return {"fc1_w": _shard(lw["up_w"], r, tp), "fc2_w": _shard(lw["down_w"], r, tp, 1)}

    def run(self, layer, h):
        if "fc1_w" in layer.quant:
            mid = mixer_ops.gelu(layer._linear(h, "fc1_w"))
        else:
            mid = ops.linear(h, layer.fc1_w, layer.sh.get("fc1_w"), act="gelu")
        return layer._linear(mid, "fc2_w")


MLPS = {m.kind: m for m in (ClampedMLP, GeluMLP)}


class TokenSide:
    """Per-layer token input: proj(gelu(gate x) * e), e the layer's part of a side embedding of the token."""

    def __init__(self, dim, layer_idx):
        self.dim, self.first = dim, layer_idx * dim

    def shard(self, lw):
        return {"side_gate_w": lw["side_gate_w"], "side_proj_w": lw["side_proj_w"], "res_side.norm_w": lw["side_norm_w"]}

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
        self.tp_rank = 0
        self.mixer = MIXERS[ls["type"]](ls["mixer"], tp_size)
        self.res1 = residual(spec.streams, W, device)
        self.qkv_w = _empty((self.mixer.rows, W), dtype, device)
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
            self.res2 = residual(spec.streams, W, device)
            self.fc1_w = _empty((self.mlp.rows, W), dtype, device)
            self.fc2_w = _empty((W, self.mlp.ff), dtype, device)
        if spec.token_side:
            self.side = TokenSide(spec.token_side, layer_idx)
            self.res_side = residual(spec.streams, W, device)
            self.side_gate_w = _empty((spec.token_side, W), dtype, device)
            self.side_proj_w = _empty((W, spec.token_side), dtype, device)

    def projection_names(self):
        return ("qkv_w", "o_w") + self.mixer.extra_projections + (("fc1_w", "fc2_w") if self.mlp else ()) + \
            (("side_gate_w", "side_proj_w") if self.side else ())

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
        if self.side:
            out.update(self.side.shard(lw))
        for q in (1, 2) if self.mlp else (1, ):
            out[f"res{q}.norm_w"] = lw[f"norm{q}_w"]
            for n in ("in", "out", "mix"):
                if f"hc{q}_{n}" in lw:
                    out[f"res{q}.{'in_' if n == 'in' else n}"] = lw[f"hc{q}_{n}"]
        return out

    def forward(self, x, pending, meta, cache, carry):
        """x: the residual, fp32. `pending`: (output, residual weights) of the sublayer before, not yet added, or the
        input of the first layer. Returns this layer's last sublayer as pending."""
        h = pending if torch.is_tensor(pending) else self.res1.enter(self.spec, x, pending)
        pending = (self._allreduce(self._linear(self.mixer.run(self, h, meta, cache, carry), "o_w")), self.res1)
        if self.mlp:
            h = self.res2.enter(self.spec, x, pending)
            pending = (self._allreduce(self.mlp.run(self, h)), self.res2)
        if self.side:
            h = self.res_side.enter(self.spec, x, pending)
            pending = (self.side.run(self, h, carry), self.res_side)
        return pending


class DSHybridModel(DSInferenceModel):
    layer_class = DSHybridLayer

    def __init__(self, spec, tp_group=None, tp_size=1, tp_rank=0, dtype=torch.bfloat16, device=None):
        super().__init__(spec, tp_group, tp_size, tp_rank, dtype, device)
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
                y, r = pending
                trace.append(r.peek(spec, x, y))
        if meta.last_idx.numel() == 0:
            return tokens.new_empty((0, spec.vocab_size), dtype=self.dtype)
        y, r = pending
        return self._logits(r.finish(self, x, y, meta.last_idx.to(torch.int32)))

    def _logits(self, h):
        return self._gather_vocab(ops.linear(h, self.lm_head, getattr(self, "lm_head_sh", None)))


def model_class(spec):
    """The model class a spec describes."""
    return DSHybridModel if spec.layer_specs else DSInferenceModel
