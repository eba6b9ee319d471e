"""Nigilorn through the framework: policy, weight loading, cache and state slots, ragged batches, scheduler, kernels — against
the plain implementation in `nigilorn_oracle.py`."""
import copy
import json

import pytest
import torch

from ...common import run_distributed
from . import nigilorn_oracle as O
from .test_vopepel import GPU, _one_thread, engine, err, feed, save, tokens  # noqa: F401

DTYPES = [pytest.param("float32", id="fp32"), pytest.param("float32", id="fp32-gpu", marks=GPU),
          pytest.param("bfloat16", id="bf16-gpu", marks=GPU)]


def model(cfg, seed, dtype):
    """Weights; 16-bit models route without near ties, so that rounding cannot pick another expert."""
    return O.random_model(cfg, seed, decisive=dtype == "bfloat16")


class Want:
    """The oracle's logits of one sequence and, per position, how far rounding the projections to bf16 moves them."""

    def __init__(self, cfg, w, ids, dtype):
        self.logits, self.dtype = O.forward(cfg, w, ids), dtype
        if dtype == "bfloat16":
            with O.Rounded():
                self.noise = self._dist(O.forward(cfg, w, ids), self.logits)

    @staticmethod
    def _dist(a, b):
        d = a.double().cpu() - b
        return (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt()

    def accepts(self, got, first=0, tol=4e-5):
        e = self._dist(got, self.logits[first:first + len(got)])
        if self.dtype == "float32":
            return e.max().item() < tol * max(1.0, self.logits.std().item())
        return e.max() < 4 * self.noise.max() and (len(e) < 30 or e.mean() < 2 * self.noise.mean())

    def shows(self, other):
        """A fault that moves the logits to `other` would not be taken for rounding."""
        d = self._dist(other, self.logits).max()
        limit = 8 * self.noise.max() if self.dtype == "bfloat16" else 1e-3
        assert d > limit, (d, limit)
        return True


def small(**kw):
    """Unequal layers: every mixer with other sizes, key and value widths that differ, partial and full rotation, every kind of
    feed-forward and none, windows below, at and across page sizes, a single group of experts and one that keeps them all, groups
    of one expert."""
    return O.config([
        O.attention_layer(heads=6, kv_heads=2, dim=16, vdim=24, size=24, rot=O.rotation(8), mlp=O.dense(40)),
        O.mamba_layer(inner=48, state=12, dt_rank=6, conv=4, mlp=O.moe(6, 2, 3, 2, 24, 40)),
        O.latent_layer(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=40, size=33, mlp=O.moe(5, 1, 1, 1, 40, 16, 1.0)),
        O.attention_layer(heads=2, kv_heads=2, dim=32, vdim=8, size=70, rot=O.rotation(32, 30.0, 1.0), scale=0.3, mlp=None),
        O.mamba_layer(inner=32, state=16, dt_rank=16, conv=3, mlp=O.dense(24)),
        O.mamba_layer(inner=40, state=5, dt_rank=3, conv=1, mlp=None),
        O.latent_layer(heads=2, dim=24, rot_dim=16, vdim=8, kv_rank=16, size=1, rot=O.rotation(16, 5e4, 8.0, 500, 32.0, 1.0),
                       mlp=O.moe(8, 3, 4, 4, 16, 8, 2.5)),
        O.attention_layer(heads=3, kv_heads=1, dim=24, vdim=16, size=16, rot=O.rotation(2), mlp=O.moe(4, 2, 4, 3, 32, 32)),
    ], **kw)


# ------------------------------------------------------------------------------------------------ whole model
@pytest.mark.parametrize("dtype", DTYPES)
def test_prompt_and_portions(tmp_path, dtype):
    """Whole prompts, token by token, and portions of several sizes (two tokens, odd ones, across page and window edges, on both
    sides of where recurrences and latent attention change kernels) give the oracle's logits at every position."""
    cfg = small()
    w = model(cfg, 1, dtype)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 150)
    want = Want(cfg, w, ids, dtype)
    for uid, cuts in enumerate(([150], [1], [2], [17, 3], [64, 64, 2, 1], [65, 1], [5, 129, 1], [16], [33], [24, 66, 1, 70])):
        assert want.accepts(feed(eng, uid, ids, cuts)), cuts
        eng.flush(uid)


@pytest.mark.parametrize("dtype", DTYPES)
def test_residual_layer_by_layer(tmp_path, dtype):
    cfg = small()
    w = model(cfg, 2, dtype)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 30)
    trace, want, rounded = [], [], []
    O.forward(cfg, w, ids, trace=want)
    with O.Rounded():
        O.forward(cfg, w, ids, trace=rounded)
    seq = eng._state_manager.get_or_create_sequence(0)
    eng._state_manager.allocate_blocks(seq, 30)
    eng._batch.clear()
    eng._batch.insert_sequence(seq, ids)
    eng._batch.finalize()
    eng.model.forward_ragged(eng._batch.input_ids(), eng._batch.meta, trace=trace)
    assert len(trace) == len(want)
    for a, b, c in zip(trace, want, rounded):
        limit = 1e-4 if dtype == "float32" else 4 * (b - c).abs().max().item()
        assert (a.double().cpu() - b).abs().max() < limit


@pytest.mark.parametrize("dtype", DTYPES)
def test_mixed_batches_and_reuse(tmp_path, dtype):
    """Unequal requests in one batch (portions beside single tokens, one pausing, one joining late), then new requests on
    the freed pages and slots: each equals itself alone."""
    cfg = small()
    w = model(cfg, 3, dtype)
    eng = engine(tmp_path, cfg, w, dtype, block=8, blocks=60, live=3)
    lens = {0: 90, 1: 41, 2: 7, 3: 180, 4: 66, 5: 1, 6: 175}
    ids = {u: tokens(cfg, n, u) for u, n in lens.items()}
    want = {u: Want(cfg, w, t, dtype) for u, t in ids.items()}
    at = {u: 0 for u in lens}
    waiting, live, step = list(lens), [], 0
    g = torch.Generator().manual_seed(0)
    sizes = [1, 2, 3, 16, 17, 90, 1, 1]
    while waiting or live:
        while waiting and len(live) < 3:
            live.append(waiting.pop(0))
        batch = [u for u in live if torch.rand(1, generator=g) < 0.8] or live[:1]
        cut = {u: min(sizes[int(torch.randint(0, 8, (1, ), generator=g))], lens[u] - at[u]) for u in batch}
        got = eng.put(batch, [ids[u][at[u]:at[u] + cut[u]] for u in batch],
                      logit_positions=[range(cut[u]) for u in batch]).float().cpu()
        row = 0
        for u in batch:
            assert want[u].accepts(got[row:row + cut[u]], at[u]), (step, u, at[u], cut[u])
            row, at[u] = row + cut[u], at[u] + cut[u]
            if at[u] == lens[u]:
                eng.flush(u)
                live.remove(u)
        step += 1
    assert eng._state_manager.free_blocks == 60 and eng._state_manager.free_slots == 3


@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens(tmp_path, dtype):
    """Sequences of one, two, three tokens: nothing before the start, in slots whose last owner left a state and a window."""
    cfg = small(eps=1e-2)
    w = model(cfg, 4, dtype)
    eng = engine(tmp_path, cfg, w, dtype, live=2)
    for n in (70, 1, 2, 3, 5):
        ids = tokens(cfg, n, n)
        want = Want(cfg, w, ids, dtype)
        for cuts in ([n], [1]):
            assert want.accepts(feed(eng, 0, ids, cuts)), (n, cuts)
            eng.flush(0)


def _asking(kind, size, heads=2, vdim=32):
    """A model of one layer in which token 10 + i asks for token i and for nothing else: its embedding is token i's turned by
    one column, and so is the query map; from there on queries and keys are the same. Positions turn little."""
    if kind == "attention":
        layer = O.attention_layer(heads=heads, kv_heads=heads, dim=32, vdim=vdim, size=size, scale=0.6,
                                  rot=O.rotation(4, 1e6, 1.2))
    else:
        layer = O.latent_layer(heads=heads, dim=32, rot_dim=8, vdim=vdim, kv_rank=48, size=size, scale=0.6,
                               rot=O.rotation(8, 1e6, 1.2))
    cfg = O.config([layer], vocab=300, width=96)
    w = O.random_model(cfg, 5)
    w["embed"][10:20] = w["embed"][:10].roll(1, -1)
    w["l0.norm1"] = torch.ones(96).bfloat16()
    m = "l0.mix."
    if kind == "attention":
        w[m + "q"] = w[m + "k"].roll(1, -1)
        w[m + "g"] *= 0.2        # (open gates)
    else:
        c = w[m + "dkv"][:48].double() * w[m + "dkv.norm"].double()[:, None]
        key = torch.cat([(w[m + "uk"].double() @ c).view(heads, 32, 96), torch.zeros(heads, 8, 96, dtype=torch.float64)], 1)
        w[m + "q"] = key.reshape(-1, 96).roll(1, -1).bfloat16()
    return cfg, w


KINDS = ["attention", "latent_attention"]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", KINDS)
def test_far_key(tmp_path, dtype, kind):
    """A single key hundreds of tokens back that dominates its query, seen from a prompt, a portion and decoding."""
    cfg, w = _asking(kind, 100000)
    eng = engine(tmp_path, cfg, w, dtype, blocks=120)
    ids = torch.cat([torch.arange(10), 20 + tokens(cfg, 579) % 280, torch.arange(10, 17)])
    want = Want(cfg, w, ids, dtype)
    other = want.logits.clone()
    other[-7:] = O.forward(cfg, w, torch.cat([ids[300:310], ids[10:]]))[-7:]
    assert want.shows(other)
    for uid, cuts in enumerate(([596], [560, 1], [301, 2], [500, 70, 26])):
        assert want.accepts(feed(eng, uid, ids, cuts)), cuts
        eng.flush(uid)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size", [70, 64, 16, 37, 130])
@pytest.mark.parametrize("kind", KINDS)
def test_window_edges(tmp_path, dtype, size, kind):
    """The asked-for key as the oldest in the window and as the one just before it, at the first and the last token of a page and
    elsewhere; from prompts, from portions that start anywhere (also far behind the first tokens), and in decoding."""
    cfg, w = _asking(kind, size)
    eng = engine(tmp_path, cfg, w, dtype, blocks=40)
    n = 3 * size + 50
    ids = 20 + tokens(cfg, n, 1) % 280
    for i, key in enumerate((15, 16, 5, size + 2, 32, size + 31, 47)):
        query = key + size - 1 + i % 2      # by turns just inside and just outside
        if query < n:
            ids[key], ids[query] = i, 10 + i
    ids[2 * size + 40], ids[3 * size + 39] = 8, 18     # inside, near the end
    ids[2 * size + 42], ids[3 * size + 42] = 9, 19     # outside
    want = Want(cfg, w, ids, dtype)
    for wrong in (size - 1, size + 1):          # an edge one token off would show
        off = copy.deepcopy(cfg)
        off["layers"][0]["mixer"]["mask"]["size"] = wrong
        assert want.shows(O.forward(off, w, ids))
    for uid, cuts in enumerate(([n], [1], [size, 2], [size + 1, 1], [2 * size - 1, 1, 1, size], [n - 20, 2], [65, 67, 66],
                                [2 * size, 90, 1])):
        assert want.accepts(feed(eng, uid, ids, cuts)), cuts
        eng.flush(uid)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_state(tmp_path, dtype):
    """Slow decays: tokens far back stay in the state; long decoding after a long prompt. Fast ones and large steps beside them."""
    cfg = O.config([O.mamba_layer(inner=40, state=12, dt_rank=8, conv=4), O.mamba_layer(inner=24, state=8, dt_rank=4, conv=2,
                                                                                        mlp=O.moe())], eps=1e-3)
    w = model(cfg, 7, dtype)
    w["l0.mix.A_log"] -= 9            # nothing is forgotten, some numbers excepted
    w["l0.mix.A_log"][:, :3] += 12
    w["l0.mix.dt.b"][:5] = 4          # steps of several units
    eng = engine(tmp_path, cfg, w, dtype)
    ids = torch.cat([tokens(cfg, 40) % 20, 20 + tokens(cfg, 290, 1) % 77])
    want = Want(cfg, w, ids, dtype)
    other = want.logits.clone()                                # the first tokens show at the end
    other[-50:] = O.forward(cfg, w, torch.cat([(ids[:40] + 1) % 20, ids[40:]]))[-50:]
    assert want.shows(other)
    for uid, cuts in enumerate(([330], [200, 1], [100, 17, 16, 2])):
        assert want.accepts(feed(eng, uid, ids, cuts)), cuts


@pytest.mark.parametrize("dtype", DTYPES[:2])
def test_every_part_shows(tmp_path, dtype):
    """The model's other branches one by one: left out of the oracle, each would move the logits by far more than the test allows."""
    cfg = small()
    w = model(cfg, 8, dtype)
    ids = tokens(cfg, 60)
    want = Want(cfg, w, ids, dtype)
    wide = lambda n: torch.full_like(w[n], 30.0)

    def without(**change):
        return O.forward(cfg, {**w, **change}, ids)

    for name in ("l0.rg1.b", "l1.rg2.b", "l2.rg2.b"):                     # gates of the residual
        assert want.shows(without(**{name: wide(name)}))
    for name in ("l0.mix.g", "l3.mix.g"):                                   # gates of the heads: all one half
        assert want.shows(without(**{name: torch.zeros_like(w[name])}))
    for name in ("l1.mlp.shared.down", "l1.mix.D", "l4.mix.conv.b", "l5.side.proj", "l2.mix.dkv.norm"):
        assert want.shows(without(**{name: torch.zeros_like(w[name])}))
    for at, key, value in ((("layers", 1, "mlp", "router"), "scale", 1.0), (("layers", 0, "mixer", "rot", "scaling"), "factor", 1.0),
                           (("layers", 0, "mixer", "rot", "scaling"), "fast", 1.0), (("layers", 2, "mixer", "rot", "scaling"), "slow", 2.0),
                           (("layers", 2, "mixer"), "scale", 0.2), (("layers", 1, "mlp", "router", "groups"), "keep", 3)):
        off = copy.deepcopy(cfg)
        d = off
        for k in at:
            d = d[k]
        assert d[key] != value
        d[key] = value
        assert want.shows(O.forward(off, w, ids)), (at, key)
    eng = engine(tmp_path, cfg, w, dtype)
    assert want.accepts(feed(eng, 0, ids, [40, 1]))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,vocab", [(200, 131), (132, 61), (37, 50)])
def test_model_widths(tmp_path, dtype, width, vocab):
    """Widths no vector or matrix tile divides."""
    cfg = O.config([O.attention_layer(heads=3, kv_heads=3, dim=20, vdim=12, size=31, rot=O.rotation(6), mlp=O.moe(7, 3, 1, 1, 27, 11)),
                    O.mamba_layer(inner=21, state=7, dt_rank=5, conv=6, mlp=O.dense(33)),
                    O.latent_layer(heads=5, dim=10, rot_dim=6, vdim=7, kv_rank=18, size=27, mlp=O.moe(9, 2, 3, 1, 45, 5))],
                   width=width, vocab=vocab, eps=1e-3, side=7)
    w = model(cfg, 16, dtype)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 90)
    want = Want(cfg, w, ids, dtype)
    for u, cuts in enumerate(([90], [40, 2], [60, 1])):
        assert want.accepts(feed(eng, u, ids, cuts)), cuts


@GPU
@pytest.mark.parametrize("attn,latent,mamba", [
    ((8, 2, 128, 128, 64, 64), (4, 56, 16, 48, 80, 75), (288, 16, 16, 4)),
    ((4, 4, 64, 96, 100, 16), (8, 128, 64, 128, 512, 33), (512, 24, 8, 4)),
    ((12, 1, 96, 64, 48, 96), (3, 40, 24, 56, 128, 64), (100, 33, 12, 2)),
    ((2, 1, 256, 256, 80, 128), (20, 24, 8, 16, 256, 20), (64, 128, 24, 3)),
    ((9, 3, 30, 20, 33, 10), (5, 20, 12, 36, 36, 90), (96, 200, 4, 4)),
    ((5, 5, 300, 40, 17, 44), (2, 96, 96, 80, 320, 130), (130, 1, 1, 5))])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sizes(tmp_path, attn, latent, mamba, dtype):
    """Head, latent and state sizes of real models and odd ones."""
    H, G, d, e, size, rot = attn
    h, n, r, v, R, win = latent
    inner, N, rank, conv = mamba
    cfg = O.config([O.attention_layer(heads=H, kv_heads=G, dim=d, vdim=e, size=size, rot=O.rotation(rot, 1e5, 4.0, 200, 8.0, 1.0)),
                    O.latent_layer(heads=h, dim=n, rot_dim=r, vdim=v, kv_rank=R, size=win),
                    O.mamba_layer(inner=inner, state=N, dt_rank=rank, conv=conv, mlp=O.moe(16, 4, 4, 2, 128, 64))],
                   width=256, vocab=130, side=32)
    w = model(cfg, 8, dtype)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 140)
    want = Want(cfg, w, ids, dtype)
    for u, cuts in enumerate(([140], [130, 1], [70, 5])):
        assert want.accepts(feed(eng, u, ids, cuts)), cuts


@GPU
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts(tmp_path, dtype):
    """Prompts long enough for every path of the expert products (few rows, lists, the library) and for contexts of which a window
    leaves only the end, in one batch with others."""
    cfg = O.config([O.attention_layer(heads=2, kv_heads=1, dim=16, vdim=16, size=300, mlp=O.moe(8, 4, 4, 2, 128, 128)),
                    O.latent_layer(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=64, size=90, mlp=O.moe(8, 4, 2, 1, 256, 64)),
                    O.mamba_layer(inner=64, state=16, dt_rank=8)], width=128)
    w = model(cfg, 21, dtype)
    eng = engine(tmp_path, cfg, w, dtype, block=64)
    ids = {u: tokens(cfg, n, u) for u, n in ((0, 700), (1, 400), (2, 5))}
    want = {u: Want(cfg, w, t, dtype) for u, t in ids.items()}
    for cuts in ([700, 400, 5], [200, 70, 1], [90, 130, 1], [30, 2, 2]):
        at = dict.fromkeys(ids, 0)
        while any(at[u] < len(t) for u, t in ids.items()):
            batch = [u for u in ids if at[u] < len(ids[u])]
            n = {u: min(cuts[u], len(ids[u]) - at[u]) for u in batch}
            got = eng.put(batch, [ids[u][at[u]:at[u] + n[u]] for u in batch], logit_positions=[range(n[u]) for u in batch])
            for u, part in zip(batch, got.split([n[u] for u in batch])):
                assert want[u].accepts(part, at[u], 1e-4), (cuts, u, at[u])
                at[u] += n[u]
        for u in ids:
            eng.flush(u)


# ------------------------------------------------------------------------------------------------ entry points
@pytest.mark.parametrize("dtype", [pytest.param("float32"), pytest.param("bfloat16", marks=GPU)])
def test_greedy_generation(tmp_path, dtype):
    """Continuous batching through `generate`: more requests than slots, a token budget that splits prompts. The oracle is
    followed along the engine's own tokens and the chosen token must be within rounding of its best."""
    cfg = small()
    w = model(cfg, 9, dtype)
    eng = engine(tmp_path, cfg, w, dtype, live=3)
    prompts = [tokens(cfg, n, 20 + n).tolist() for n in (5, 33, 1, 60, 18)]
    outs = eng.generate(prompts, max_new_tokens=9, token_budget=24)
    for p, o in zip(prompts, outs):
        assert len(o) == 9
        lg = O.forward(cfg, w, p + o[:-1])[len(p) - 1:]
        for row, tok in zip(lg, o):
            assert row.max() - row[tok] <= (1e-4 if dtype == "float32" else 0.15) * row.std()
    assert eng._state_manager.free_slots == 3 and not eng._state_manager.tracked_sequences
    again = eng.generate(prompts[:2], max_new_tokens=9, eos_token_id=outs[0][2])
    if dtype == "float32":
        assert again[0] == outs[0][:outs[0].index(outs[0][2]) + 1]
    a, b = (eng.generate(prompts[:2], max_new_tokens=5, do_sample=True, temperature=0.8, top_k=20, top_p=0.9, seed=3)
            for _ in range(2))
    assert a == b


def test_geometry_and_pools(tmp_path):
    """Keys and values only where a layer attends (latents as one row), a state where it has one; pool sizes count both."""
    from deepspeedsyclsupport_amd.inference.kv_cache import BlockedKVCache
    cfg = small()
    eng = engine(tmp_path, cfg, O.random_model(cfg, 9), "float32")
    c = eng.model.cache
    assert c.k[1] is None and tuple(c.state[1]["state"].shape) == (4, 48, 12) and tuple(c.state[1]["conv"].shape) == (4, 3, 48)
    assert tuple(c.state[5]["state"].shape) == (4, 40, 8) and set(c.state[5]) == {"state"} and c.state[0] is None
    assert tuple(c.k[0].shape[1:]) == (2, 16, 16) and tuple(c.v[0].shape[1:]) == (2, 16, 24)
    assert tuple(c.k[2].shape[1:]) == (1, 16, 48) and c.v[2].shape[3] == 0
    assert c.state[1]["state"].dtype == torch.float32
    assert c.bytes() == 64 * BlockedKVCache.block_bytes(eng.model.kv_geometry(), 16, torch.float32) + \
        4 * BlockedKVCache.slot_bytes(eng.model.state_geometry())


def test_serialize_round_trip(tmp_path):
    from deepspeedsyclsupport_amd.inference.v2 import build_engine_from_ds_checkpoint
    cfg = small()
    eng = engine(tmp_path, cfg, O.random_model(cfg, 10), "float32")
    ids = tokens(cfg, 40)
    a = eng.put([0], [ids])
    eng.serialize(str(tmp_path / "ds"))
    eng2 = build_engine_from_ds_checkpoint(str(tmp_path / "ds"), eng._config)
    assert type(eng2.model) is type(eng.model)
    assert torch.equal(eng2.put([0], [ids]).cpu(), a.cpu())


def test_bad_checkpoints(tmp_path):
    cfg = small()
    w = O.random_model(cfg, 11)
    for lacking in ("l0.mix.g", "l2.mix.dkv.norm", "l1.mlp.e3.up", "l1.mlp.shared.down", "l2.mlp.router", "l4.rg2.b", "l5.norm1b",
                    "l1.mix.A_log", "side.embed"):
        with pytest.raises(RuntimeError, match="not fully initialized"):
            engine(tmp_path, cfg, {k: v for k, v in w.items() if k != lacking}, "float32")
    for extra in ("l3.norm2", "l1.mlp.e0.gate", "l2.mix.sink", "l2.mix.uq", "l0.mix.q.b", "l0.mlp.router"):
        with pytest.raises(ValueError, match="Cannot find container"):
            engine(tmp_path, cfg, {**w, extra: torch.zeros(64)}, "float32")
    for name, t in (("l0.mix.k", torch.zeros(31, 64)), ("l1.mix.x", torch.zeros(29, 48)), ("l1.mlp.shared.up", torch.zeros(39, 64)),
                    ("l0.rg1", torch.zeros(63, 64)), ("l1.mix.dt.b", torch.zeros(47)), ("l2.mlp.router", torch.zeros(4, 64))):
        with pytest.raises((ValueError, RuntimeError), match="by the configuration|invalid for input|size"):
            engine(tmp_path, cfg, {**w, name: t}, "float32")
    for change in (lambda c: c["layers"][0].update(type="something else"), lambda c: c["layers"][0]["mlp"].update(kind="gelu")):
        bad = copy.deepcopy(cfg)
        change(bad)
        with pytest.raises(NotImplementedError):
            engine(tmp_path, bad, w, "float32")
    for path, value in ((("layers", 0, "mixer", "kv_heads"), 4), (("layers", 0, "mixer", "rot", "dims"), 18),
                        (("layers", 2, "mixer", "rot", "dims"), 10), (("layers", 1, "mlp", "router", "groups", "count"), 4),
                        (("layers", 1, "mlp", "router", "top"), 5)):
        bad = copy.deepcopy(cfg)
        at = bad
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        with pytest.raises(ValueError):
            engine(tmp_path, bad, w, "float32")


def test_parts_in_other_models(tmp_path):
    """Its mechanisms stand in other designs too: a gated sandwich residual around mixers that want whole rows, rotation by halves
    in windowed attention, latent attention with a query latent and a window."""
    from deepspeedsyclsupport_amd.inference.model_implementations.hybrid import DSHybridModel
    from deepspeedsyclsupport_amd.inference.model_implementations.transformer import DSModelSpec
    from deepspeedsyclsupport_amd.inference.v2 import AllocationMode, InferenceEngineV2, RaggedInferenceEngineConfig
    rot = {"base": 100.0, "dims": 8}
    layers = ({"type": "delta", "mixer": {"heads": 2, "kv_heads": 1, "dim": 8, "vdim": 8, "conv": 3},
               "mlp": {"kind": "dense", "ff": 24, "limit": 7.0}},
              {"type": "window_attention", "mixer": {"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 8, "scale": 0.3, "rot": rot,
                                                     "mask": {"size": 9}}, "mlp": {"kind": "gelu", "ff": 20}},
              {"type": "latent_attention", "mixer": {"heads": 2, "dim": 8, "rot_dim": 8, "vdim": 8, "kv_rank": 16, "q_rank": 16,
                                                     "scale": 0.3, "rot": rot, "mask": {"size": 11}},
               "mlp": {"kind": "routed", "expert": {"ff": 16}, "router": {"experts": 4, "top": 2}}})
    spec = DSModelSpec(arch="test", vocab_size=50, hidden_size=32, num_layers=3, num_heads=4, num_kv_heads=2, intermediate_size=0,
                       norm="rms", pos="none", residual="sandwich", residual_gate=True, layer_specs=layers)
    outs = []
    for device in ["cpu"] + (["cuda"] if torch.cuda.is_available() else []):
        m = DSHybridModel(spec, dtype=torch.float32, device=torch.device(device))
        g = torch.Generator().manual_seed(0)
        with torch.no_grad():
            for p in m.parameters():
                if p.dim() > 1:
                    p.copy_(torch.randn(p.shape, generator=g) * p.shape[-1]**-0.5)
        eng = InferenceEngineV2(m, RaggedInferenceEngineConfig(
            state_manager={"memory_config": {"mode": AllocationMode.ALLOCATE, "size": 8}, "max_tracked_sequences": 2,
                           "max_ragged_sequence_count": 2, "max_context": 128}, kv_cache={"block_size": 16}))
        ids = torch.arange(45) * 7 % 50
        outs += [feed(eng, u, ids, cuts) for u, cuts in enumerate(([45], [30, 1]))]
    for o in outs[1:]:
        assert err(o, outs[0]) < 1e-4 and outs[0].std() > 0.1


@GPU
def test_weight_only_int8(tmp_path):
    """The framework's weight-only quantisation reaches these layers' projections too."""
    cfg = O.config([O.attention_layer(heads=4, kv_heads=2, dim=64, vdim=64, mlp=O.moe(ff=64, shared=64)),
                    O.mamba_layer(inner=128, state=24, dt_rank=16, mlp=O.dense(64)),
                    O.latent_layer(heads=4, dim=32, rot_dim=16, vdim=64, kv_rank=64, mlp=O.dense(128))], width=256, vocab=128,
                   side=64)
    w = model(cfg, 12, "bfloat16")
    eng = engine(tmp_path, cfg, w, "bfloat16")
    ids = tokens(cfg, 40)
    want = O.forward(cfg, w, ids)
    eng.model.quantize_weights(8)
    assert err(feed(eng, 0, ids, [30, 1]), want) < 0.2 * want.std()


def _tp_run(path, ids, want):
    from deepspeedsyclsupport_amd.inference.v2 import (AllocationMode, RaggedInferenceEngineConfig, build_hf_engine)
    torch.set_num_threads(1)
    conf = RaggedInferenceEngineConfig(
        state_manager={"memory_config": {"mode": AllocationMode.ALLOCATE, "size": 16}, "max_tracked_sequences": 2,
                       "max_ragged_sequence_count": 2, "max_context": 256}, kv_cache={"block_size": 16},
        tensor_parallel={"tp_size": 2})
    eng = build_hf_engine(path, conf, dtype=torch.float32)
    got = torch.cat([eng.put([0], [ids[:40]], logit_positions=[range(40)]),
                     eng.put([0], [ids[40:]], logit_positions=[range(10)])])
    assert err(got, want) < 5e-5


@pytest.mark.skipif(torch.cuda.is_available(), reason="ranks exchange host tensors")
def test_tensor_parallel(tmp_path):
    """Heads, experts and vocabulary over two ranks; recurrences run whole on each and hand on their share."""
    cfg = O.config([O.attention_layer(heads=6, kv_heads=2, mlp=O.moe(ff=24)), O.mamba_layer(mlp=O.dense()),
                    O.latent_layer(heads=4, mlp=O.moe(5, 2, 1, 1, 16, 8))])
    w = O.random_model(cfg, 15)
    ids = tokens(cfg, 50)
    run_distributed(_tp_run, 2, save(tmp_path / "m", cfg, w), ids, O.forward(cfg, w, ids))


# ------------------------------------------------------------------------------------------------ trace replay
def test_trace_replay(tmp_path):
    from deepspeedsyclsupport_amd.inference.v2.trace import TraceRunner, trace_engine
    cfg = small()
    w = O.random_model(cfg, 13)
    eng = trace_engine(save(tmp_path / "m", cfg, w), torch.float32, 192)
    a, b = tokens(cfg, 70, 1).tolist(), tokens(cfg, 90, 2).tolist()
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:40], "want": [3, 39]}, {"id": "b", "tokens": b[:1], "want": []}],
              "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[1:90], "want": [0, 88]}, {"id": "a", "tokens": a[40:41],
                                                                                      "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[41:], "want": []}], "end": ["a"]}]
    said = []
    TraceRunner(eng, str(tmp_path)).run([json.dumps(s) for s in steps], said.append)
    assert said == ["done 0", "done 1", "done 2"] and not (tmp_path / "2.f32").exists()
    la, lb = O.forward(cfg, w, a), O.forward(cfg, w, b)

    def read(i):
        return torch.frombuffer(bytearray((tmp_path / f"{i}.f32").read_bytes()), dtype=torch.float32).view(-1, cfg["vocab"])

    assert err(read(0), la[[3, 39]]) < 5e-5
    assert err(read(1), torch.stack([lb[1], lb[89], la[40]])) < 5e-5
    assert eng._state_manager.free_blocks == 3 and eng._state_manager.free_slots == 4
