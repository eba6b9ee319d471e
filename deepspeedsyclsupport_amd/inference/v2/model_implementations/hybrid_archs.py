"""Containers and policies of the hybrid decoders (`inference/model_implementations/hybrid.py`): checkpoints that are
config.json + model.safetensors in this package's own layout, with the layers listed one by one in the config.

A layer's container is assembled from the tensors its kind has: the mixer's, the feed-forward's if it has one, the
norms and, for models with residual streams, the mixing matrices."""
from types import SimpleNamespace

import torch

from ...model_implementations.hybrid import DSHybridModel, ParallelMixer
from ...model_implementations.transformer import DSModelSpec
from .inference_policy_base import ContainerMap, InferenceV2Policy, register
from .layer_container_base import LayerContainer
from .parameter_base import ParamList, ParameterBase, single

_MIXER_TENSORS = {  # checkpoint name below `<layer>.mix.` -> canonical key
    "attention": {"q": "q_w", "k": "k_w", "v": "v_w", "o": "o_w", "q.norm": "q_norm", "k.norm": "k_norm"},
    "delta": {"q": "q_w", "k": "k_w", "v": "v_w", "g": "g_w", "b": "b_w", "a": "a_w", "o": "o_w", "q.conv": "q_conv",
              "k.conv": "k_conv", "v.conv": "v_conv", "A_log": "a_log", "dt_bias": "dt_bias", "norm": "head_norm"},
    "latent_attention": {"dq": "dq_w", "dq.norm": "q_norm", "uq": "uq_w", "dkv": "dkv_w", "dkv.norm": "kv_norm",
                         "uk": "uk_w", "uv": "uv_w", "sink": "sink", "o": "o_w"},
    "window_attention": {"q": "q_w", "k": "k_w", "v": "v_w", "g": "g_w", "o": "o_w"},
    "mamba1": {"in": "in_w", "conv": "conv_w", "conv.b": "conv_b", "x": "x_w", "dt": "dt_w", "dt.b": "dt_bias", "A_log": "a_log",
               "D": "skip", "o": "o_w"},
    "mamba2": {"in": "in_w", "conv": "conv_w", "conv.b": "conv_b", "dt_bias": "dt_bias", "A_log": "a_log", "D": "skip",
               "norm": "head_norm", "o": "o_w"},
    "lightning": {"q": "q_w", "k": "k_w", "v": "v_w", "g": "g_w", "o": "o_w", "norm": "head_norm"},
    "rotary_attention": {"q": "q_w", "k": "k_w", "v": "v_w", "q.b": "q_b", "k.b": "k_b", "v.b": "v_b", "q.norm": "q_norm",
                         "k.norm": "k_norm", "o": "o_w"},
    "matrix_memory": {"q": "q_w", "k": "k_w", "v": "v_w", "g": "g_w", "i": "i_w", "i.b": "i_b", "f": "f_w", "f.b": "f_b",
                      "norm": "head_norm", "o": "o_w"},
    "retention": {"q": "q_w", "k": "k_w", "v": "v_w", "g": "g_w", "o": "o_w"},
}
_MIXER_TENSORS["parallel"] = {f"{side}.{n}": f"{side}_{key}" for side, cls in ParallelMixer.sides
                              for n, key in _MIXER_TENSORS[cls.kind].items()}
_MLP_TENSORS = {"dense": {"gate": "gate_w", "up": "up_w", "down": "down_w"}, "gelu": {"up": "up_w", "down": "down_w"},
                "silu_glu": {"gate": "gate_w", "up": "up_w", "down": "down_w"}, "routed": {"router": "router_w"}}
_EXPERT_TENSORS = ("gate", "up", "down")   # (a plain expert has no gate)
_SANDWICH_TENSORS = {"norm{}b": "post{}_w", "rg{}": "rg{}_w", "rg{}.b": "rg{}_b"}
_SIDE_TENSORS = {"side.gate": "side_gate_w", "side.proj": "side_proj_w", "side.norm": "side_norm_w"}


class _HybridContainer(LayerContainer):
    """A container that names every tensor it is made of: all must come, except those in `may_lack`."""
    may_lack = ()

    @property
    def is_initialized(self):
        return not self.missing()

    def missing(self):
        return [name for name, p in self._params.items() if not p.complete and name not in self.may_lack]


def _stacked(key, count):
    """A parameter of `count` tensors that are stacked under `key`."""

    class _Stacked(ParameterBase):
        params: ParamList("count")

        def __init__(self, model=None, name=None):
            super().__init__(SimpleNamespace(count=count), name)

        def finalize(self):
            return {key: torch.stack(list(self.params))}

    return _Stacked


def container(name, tensors, may_lack=(), stacked=None, count=0):
    """A container class for {checkpoint tensor: canonical key}; `stacked`: the same for lists of `count` tensors, the index
    being the `*` of the name."""
    lists = stacked or {}
    return type(name, (_HybridContainer, ), {
        "__annotations__": {**{key: single(key) for key in tensors.values()}, **{key: _stacked(key, count)
                                                                                for key in lists.values()}},
        "PARAM_MAPPING": {src: f"{key}.params" for src, key in {**tensors, **lists}.items()}, "may_lack": may_lack})


def _mixer_tensors(layer):
    tensors, mx = dict(_MIXER_TENSORS[layer["type"]]), layer["mixer"]
    if mx.get("v_mix"):
        tensors["vmix"] = "vmix"
    if layer["type"] == "latent_attention":
        if not mx.get("q_rank"):   # queries straight from the input
            tensors = {n: key for n, key in tensors.items() if n not in ("dq", "dq.norm", "uq")}
            tensors["q"] = "q_w"
        if not mx.get("sink", True):
            del tensors["sink"]
    return tensors


def layer_container(layer, streams=False, may_lack=(), side=False, sandwich=False):
    """Container class of one entry of the spec's layer list. `sandwich`: norms on the sublayers' outputs too, and gates."""
    if layer["type"] not in _MIXER_TENSORS:
        raise NotImplementedError(f"no mixer {layer['type']!r}")
    tensors = {f"mix.{n}": key for n, key in _mixer_tensors(layer).items()}
    lists, count = {}, 0
    if layer.get("mlp"):
        if layer["mlp"].get("kind") not in _MLP_TENSORS:
            raise NotImplementedError(f"no feed-forward {layer['mlp'].get('kind')!r}")
        if layer["mlp"]["kind"] == "routed":
            names = _EXPERT_TENSORS[0 if layer["mlp"].get("act", "silu_glu") == "silu_glu" else 1:]
            lists, count = {f"mlp.e*.{n}": f"experts_{n}" for n in names}, layer["mlp"]["router"]["experts"]
            if layer["mlp"].get("shared"):
                tensors.update({f"mlp.shared.{n}": f"shared_{n}" for n in names})
        tensors.update({f"mlp.{n}": key for n, key in _MLP_TENSORS[layer["mlp"]["kind"]].items()})
    for q in (1, 2) if layer.get("mlp") else (1, ):
        tensors[f"norm{q}"] = f"norm{q}_w"
        if streams:
            tensors.update({f"hc{q}.{n}": f"hc{q}_{n}" for n in ("in", "out", "mix")})
        if sandwich:
            tensors.update({n.format(q): key.format(q) for n, key in _SANDWICH_TENSORS.items()})
    if side:
        tensors.update(_SIDE_TENSORS)
    return container("HybridLayerContainer", tensors, may_lack, lists, count)


def _renamed(layers, kinds):
    """A config's layers with its names of feed-forwards replaced by the package's ({config's: package's}, no others)."""
    for i, la in enumerate(layers):
        if la.get("mlp") and la["mlp"].get("kind") not in kinds:
            raise NotImplementedError(f"layer {i}: no feed-forward {la['mlp'].get('kind')!r}")
    return [{**la, "mlp": {**la["mlp"], "kind": kinds[la["mlp"]["kind"]]} if la.get("mlp") else None} for la in layers]


_TOP_TENSORS = {"embed": "embed", "final.norm": "norm_w", "head": "lm_head"}
TopContainer = container("HybridTopContainer", _TOP_TENSORS)
TiedTopContainer = container("HybridTiedTopContainer", {n: k for n, k in _TOP_TENSORS.items() if k != "lm_head"})
SideTopContainer = container("HybridSideTopContainer", {**_TOP_TENSORS, "side.embed": "side_embed"})


@register
class VopepelPolicy(InferenceV2Policy):
    """Vopepel: gated-delta-rule and chunked softmax-attention layers over several residual streams."""
    model_types = ("vopepel", )
    model_class = DSHybridModel

    def spec(self):
        c = self._model_config
        attn = [la["mixer"] for la in c.layers if la["type"] == "attention"]
        first = (attn or [la["mixer"] for la in c.layers])[0]
        return DSModelSpec(arch="vopepel", vocab_size=c.vocab, hidden_size=c.width, num_layers=len(c.layers),
                           num_heads=first["heads"], num_kv_heads=first["kv_heads"], head_dim=first["dim"],
                           intermediate_size=max([la["mlp"]["ff"] for la in c.layers if la.get("mlp")], default=0),
                           norm="ln", norm_bias=False, norm_eps=float(c.norm["eps"]), pos="none",
                           layer_specs=tuple(c.layers), streams=int(getattr(c, "streams", None) or 1),
                           residual_mult=float(getattr(c, "residual_mult", 1.0)))

    def build_container_map(self):
        c = self._model_config
        cmap = ContainerMap()
        streams = bool(getattr(c, "streams", None))
        # the first value-mixing layer only lends its values: it has no use for a mixing weight
        first = next((i for i, la in enumerate(c.layers) if la["mixer"].get("v_mix")), None)
        cmap.set_transformer_params("l", [layer_container(la, streams, ("vmix", ) if i == first else ())(self._view)
                                          for i, la in enumerate(c.layers)], sep="")
        cmap.set_non_transformer_params(TopContainer(self._view))
        return cmap


@register
class PerelornPolicy(InferenceV2Policy):
    """Perelorn: state-space, linear-attention and latent-attention layers under norms on the sublayers' outputs, with a
    token-side input in every layer."""
    model_types = ("perelorn", )
    model_class = DSHybridModel

    def layers(self):
        """The config's layers in the spec's terms: its "dense" feed-forward is the ungated gelu one."""
        return _renamed(self._model_config.layers, {"dense": "gelu"})

    def spec(self):
        c = self._model_config
        first = next((la["mixer"] for la in c.layers if la["type"] == "latent_attention"), c.layers[0]["mixer"])
        return DSModelSpec(arch="perelorn", vocab_size=c.vocab, hidden_size=c.width, num_layers=len(c.layers),
                           num_heads=first["heads"], num_kv_heads=first["heads"], head_dim=first["vdim"],
                           intermediate_size=max([la["mlp"]["ff"] for la in c.layers if la.get("mlp")], default=0),
                           norm="rms", norm_eps=float(c.norm["eps"]), pos="none", layer_specs=tuple(self.layers()),
                           residual="post_norm", token_side=int(c.token_side["dim"]), logit_scale=float(c.logit_scale))

    def build_container_map(self):
        cmap = ContainerMap()
        cmap.set_transformer_params("l", [layer_container(la, side=True)(self._view) for la in self.layers()], sep="")
        cmap.set_non_transformer_params(SideTopContainer(self._view))
        return cmap


@register
class LefisunPolicy(InferenceV2Policy):
    """Lefisun: retention layers and layers of chunked rotary attention beside a matrix memory, routed experts, one fp32 residual
    with norms on the sublayers' inputs, the embedding table as output."""
    model_types = ("lefisun", )
    model_class = DSHybridModel

    def layers(self):
        """The config's layers in the spec's terms."""
        return _renamed(self._model_config.layers, {"moe": "routed"})

    def spec(self):
        c, layers = self._model_config, self.layers()
        first = next((la["mixer"]["left"] for la in layers if la["type"] == "parallel"), layers[0]["mixer"])
        return DSModelSpec(arch="lefisun", vocab_size=c.vocab, hidden_size=c.width, num_layers=len(c.layers),
                           num_heads=first["heads"], num_kv_heads=first.get("kv_heads", first["heads"]), head_dim=first["dim"],
                           intermediate_size=max([la["mlp"]["expert"]["ff"] for la in layers if la["mlp"] and "expert" in
                                                  la["mlp"]], default=0),
                           norm="rms", norm_eps=float(c.norm["eps"]), pos="none", tie_embeddings=True,
                           layer_specs=tuple(layers), residual="pre_norm", embed_scale=float(c.embedding["scale"]))

    def build_container_map(self):
        cmap = ContainerMap()
        cmap.set_transformer_params("l", [layer_container(la)(self._view) for la in self.layers()], sep="")
        cmap.set_non_transformer_params(TiedTopContainer(self._view))
        return cmap


@register
class NigilornPolicy(InferenceV2Policy):
    """Nigilorn: selective state spaces, windowed attention and windowed latent attention between norms on the sublayers' inputs
    and gated outputs, dense layers and mixtures of plain experts beside a shared one, a token-side input in every layer."""
    model_types = ("nigilorn", )
    model_class = DSHybridModel

    def layers(self):
        """The config's layers in the spec's terms, with what the design fixes: rotation of neighbours and its scaling, no sinks,
        routing by sigmoids, squared-relu experts."""
        out = []
        for i, la in enumerate(_renamed(self._model_config.layers, {"dense": "silu_glu", "moe": "routed"})):
            kinds = {"attention": "window_attention", "latent_attention": "latent_attention", "mamba1": "mamba1"}
            if la["type"] not in kinds:
                raise NotImplementedError(f"layer {i}: no mixer {la['type']!r}")
            mx, ml = dict(la["mixer"]), la["mlp"]
            if "rot" in mx:
                mx["rot"] = {**mx["rot"], "pairs": "neighbours"}
                if mx["rot"].get("scaling"):
                    mx["rot"]["scaling"] = {**mx["rot"]["scaling"], "type": "yarn"}
            if la["type"] == "latent_attention":
                mx["sink"] = False
            if ml and ml["kind"] == "routed":
                groups = ml["router"].get("groups") or {}
                ml = {**ml, "act": "relu2", "router": {**ml["router"], "score": "sigmoid", "groups": {**groups, "best": 2}}}
            out.append({"type": kinds[la["type"]], "mixer": mx, "mlp": ml})
        return out

    def spec(self):
        c, layers = self._model_config, self.layers()
        first = next((la["mixer"] for la in layers if la["type"] == "window_attention"), {"heads": 1, "vdim": c.width})
        widths = [la["mlp"].get("ff") or la["mlp"]["expert"]["ff"] for la in layers if la["mlp"]]
        return DSModelSpec(arch="nigilorn", vocab_size=c.vocab, hidden_size=c.width, num_layers=len(c.layers),
                           num_heads=first["heads"], num_kv_heads=first.get("kv_heads", first["heads"]), head_dim=first["vdim"],
                           intermediate_size=max(widths, default=0), norm="rms", norm_eps=float(c.norm["eps"]), pos="none",
                           layer_specs=tuple(layers), residual="sandwich", residual_gate=True,
                           token_side=int(c.token_side["dim"]))

    def build_container_map(self):
        cmap = ContainerMap()
        cmap.set_transformer_params("l", [layer_container(la, side=True, sandwich=True)(self._view) for la in self.layers()],
                                    sep="")
        cmap.set_non_transformer_params(SideTopContainer(self._view))
        return cmap
