"""Lefisun through the framework: policy, weight loading, cache and state slots, ragged batches, scheduler, kernels — against
the plain implementation in `lefisun_oracle.py`."""
import json

import pytest
import torch

from ...common import run_distributed
from . import lefisun_oracle as O
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
    """Unequal layers: every mixer with other sizes, key and value widths that differ, with and without a feed-forward, chunks
    below, at and across page sizes, a single group of experts and one that keeps them all."""
    return O.config([
        O.parallel_layer(heads=6, kv_heads=2, dim=16, vdim=24, size=24, rot=8, r_heads=3, r_dim=24, r_vdim=16,
                         mlp=O.moe(6, 2, 3, 2, 24)),
        O.retention_layer(heads=3, dim=16, vdim=24, mlp=None),
        O.parallel_layer(heads=2, kv_heads=2, dim=32, vdim=8, size=70, rot=32, base=30.0, factor=1.0, scale=0.3, left_scale=1.0,
                         right_scale=1.3, r_heads=2, r_dim=8, r_vdim=40, cap=2.0, mlp=O.moe(5, 1, 1, 1, 40)),
        O.parallel_layer(heads=4, kv_heads=1, dim=24, vdim=16, size=1, rot=0, r_heads=1, r_dim=40, r_vdim=8, mlp=None),
        O.retention_layer(heads=2, dim=40, vdim=16, rot=16, decay=[1.0, 0.2], base=100.0, mlp=O.moe(8, 3, 4, 4, 16)),
        O.parallel_layer(heads=3, kv_heads=3, dim=8, vdim=8, size=16, rot=4, r_heads=4, r_dim=16, r_vdim=16,
                         mlp=O.moe(8, 2, 4, 1, 32)),
    ], **kw)


# ------------------------------------------------------------------------------------------------ whole model
@pytest.mark.parametrize("dtype", DTYPES)
def test_prompt_and_portions(tmp_path, dtype):
    """Whole prompts, token by token, and portions of several sizes (two tokens, odd ones, across page, mask-chunk and
    state-chunk edges, on both sides of where recurrences change kernels) give the oracle's logits at every position."""
    cfg = small()
    w = model(cfg, 1, dtype)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 150)
    want = Want(cfg, w, ids, dtype)
    for uid, cuts in enumerate(([150], [1], [2], [17, 3], [64, 64, 2, 1], [65, 1], [5, 129, 1], [16], [33], [24, 46, 1, 70])):
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
    lens = {0: 90, 1: 41, 2: 7, 3: 180, 4: 66, 5: 1, 6: 75}
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
    """Sequences of one, two, three tokens: nothing before the start, in slots whose last owner left a state, a normaliser and
    a maximum."""
    cfg = small(eps=1e-2, scale=0.4)
    w = model(cfg, 4, dtype)
    eng = engine(tmp_path, cfg, w, dtype, live=2)
    for n in (70, 1, 2, 3, 5):
        ids = tokens(cfg, n, n)
        want = Want(cfg, w, ids, dtype)
        for cuts in ([n], [1]):
            assert want.accepts(feed(eng, 0, ids, cuts)), (n, cuts)
            eng.flush(0)


def _asking(size, dtype, heads=2, vdim=32):
    """A model of one layer in which token 10 + i asks for token i and for nothing else: its embedding is token i's turned by
    one column, and so is the query map; from there on queries and keys are the same. Positions hardly turn anything."""
    cfg = O.config([O.parallel_layer(heads=heads, kv_heads=heads, dim=32, vdim=vdim, size=size, rot=8, factor=1e7, scale=0.6,
                                     left_scale=1.5, right_scale=0.1, r_heads=1, r_dim=8, r_vdim=8)], vocab=300, width=96)
    w = O.random_model(cfg, 5)
    w["embed"][10:20] = w["embed"][:10].roll(1, -1)
    w["l0.norm1"] = torch.ones(96).bfloat16()
    p = "l0.mix.left."
    w[p + "q"], w[p + "q.norm"] = w[p + "k"].roll(1, -1), w[p + "k.norm"].clone()
    w[p + "q.b"], w[p + "k.b"] = (torch.zeros_like(w[p + "k.b"]) for _ in range(2))
    return cfg, w


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_key(tmp_path, dtype):
    """A single key hundreds of tokens back that dominates its query, seen from a prompt, a portion and decoding."""
    cfg, w = _asking(100000, dtype)
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
@pytest.mark.parametrize("size", [70, 64, 16, 37])
def test_chunk_edges(tmp_path, dtype, size):
    """The asked-for key as the first of the query's chunk, the last of the one before (not to be seen), and the first and the
    last of a page; queries as the first and the last token of a chunk."""
    cfg, w = _asking(size, dtype)
    eng = engine(tmp_path, cfg, w, dtype, blocks=40)
    ids = 20 + tokens(cfg, 4 * size + 3, 1) % 280
    pairs = [(size, 2 * size - 1), (size - 1, size + 1), (2 * size, 2 * size + 2), (2 * size - 2, 2 * size), (3 * size + 1,
             4 * size - 1), (3 * size, 4 * size)]
    for i, (key, query) in enumerate(pairs):
        ids[key], ids[query] = i, 10 + i
    want = Want(cfg, w, ids, dtype)
    for wrong in (size - 1, size + 1):          # an edge one token off would show
        off = json.loads(json.dumps(cfg))
        off["layers"][0]["mixer"]["left"]["mask"]["size"] = wrong
        assert want.shows(O.forward(off, w, ids))
    for uid, cuts in enumerate(([len(ids)], [1], [size, 2], [size + 1, 1], [2 * size - 1, 1, 1, size], [3 * size - 1, 2])):
        assert want.accepts(feed(eng, uid, ids, cuts)), cuts
        eng.flush(uid)


@pytest.mark.parametrize("dtype", DTYPES)
def test_sink_shows(tmp_path, dtype):
    """Scores far below zero leave most of the weight to the sink: without it the outputs would be many times as large."""
    cfg = O.config([O.parallel_layer(heads=4, kv_heads=2, size=50, scale=0.3, rot=0, left_scale=2.0, right_scale=0.2)])
    w = O.random_model(cfg, 6)
    p = "l0.mix.left."
    w[p + "k"], w[p + "q"] = w[p + "k"] * 0.3, w[p + "q"] * 0.3
    w[p + "q.b"] = 2 * torch.ones(64).bfloat16()
    w[p + "k.b"] = -2 * torch.ones(32).bfloat16()
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 120)
    want = Want(cfg, w, ids, dtype)
    held, O.chunked_attention = O.chunked_attention, _no_sink
    try:
        assert want.shows(O.forward(cfg, w, ids))
    finally:
        O.chunked_attention = held
    for uid, cuts in enumerate(([120], [30, 1], [100, 15, 2])):
        assert want.accepts(feed(eng, uid, ids, cuts)), cuts


def _no_sink(q, k, v, scale, chunk):
    return torch.stack([torch.softmax((k[i // chunk * chunk:i + 1] @ q[i]) * scale, -1) @ v[i // chunk * chunk:i + 1]
                        for i in range(len(q))])


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_state(tmp_path, dtype):
    """Slow decays and open forget gates: tokens far back stay in the states; long decoding after a long prompt."""
    cfg = O.config([O.parallel_layer(heads=2, kv_heads=1, size=20, left_scale=0.3, right_scale=1.5, r_heads=3, r_dim=24, r_vdim=40,
                                     cap=9.0),
                    O.retention_layer(heads=2, dim=24, vdim=8, decay=[0.9999, 0.97], rot=8, mlp=O.moe())], eps=1e-3)
    w = model(cfg, 7, dtype)
    w["l0.mix.right.f.b"] += 6        # one head forgets nothing, one a little, one nearly everything
    w["l0.mix.right.f.b"][1] -= 5
    w["l0.mix.right.f.b"][2] = -5
    w["l0.mix.right.i"][0] *= 6       # and the running maximum rises late
    eng = engine(tmp_path, cfg, w, dtype)
    ids = torch.cat([tokens(cfg, 40) % 20, 20 + tokens(cfg, 290, 1) % 77])
    want = Want(cfg, w, ids, dtype)
    other = want.logits.clone()                                # the first tokens show at the end
    other[-50:] = O.forward(cfg, w, torch.cat([(ids[:40] + 1) % 20, ids[40:]]))[-50:]
    assert want.shows(other)
    for uid, cuts in enumerate(([330], [200, 1], [100, 17, 16, 2])):
        assert want.accepts(feed(eng, uid, ids, cuts)), cuts


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,vocab", [(200, 131), (132, 61), (37, 50)])
def test_model_widths(tmp_path, dtype, width, vocab):
    """Widths no vector or matrix tile divides."""
    cfg = O.config([O.parallel_layer(heads=3, kv_heads=3, dim=20, vdim=12, size=31, rot=6, r_heads=3, r_dim=18, r_vdim=10,
                                     mlp=O.moe(7, 3, 1, 1, 27)),
                    O.retention_layer(heads=2, dim=10, vdim=5, rot=6, mlp=O.moe(9, 2, 3, 1, 45))], width=width, vocab=vocab,
                   eps=1e-3)
    w = model(cfg, 16, dtype)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 90)
    want = Want(cfg, w, ids, dtype)
    for u, cuts in enumerate(([90], [40, 2], [60, 1])):
        assert want.accepts(feed(eng, u, ids, cuts)), cuts


@GPU
@pytest.mark.parametrize("left,scan", [((8, 2, 128, 128, 64, 64), (4, 128, 64)), ((4, 4, 64, 96, 100, 16), (2, 256, 128)),
                                       ((12, 1, 96, 64, 48, 96), (3, 64, 96)), ((2, 1, 256, 256, 80, 128), (1, 96, 256)),
                                       ((6, 3, 30, 20, 33, 10), (2, 320, 40))])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sizes(tmp_path, left, scan, dtype):
    """Head sizes of real models and odd ones."""
    H, G, d, e, size, rot = left
    h, n, v = scan
    cfg = O.config([O.parallel_layer(heads=H, kv_heads=G, dim=d, vdim=e, size=size, rot=rot, r_heads=h, r_dim=n, r_vdim=v),
                    O.retention_layer(heads=h, dim=n // 2, vdim=v, mlp=O.moe(16, 4, 4, 2, 128))], width=256, vocab=130)
    w = model(cfg, 8, dtype)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 140)
    want = Want(cfg, w, ids, dtype)
    for u, cuts in enumerate(([140], [130, 1], [70, 5])):
        assert want.accepts(feed(eng, u, ids, cuts)), cuts


@GPU
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts(tmp_path, dtype):
    """Prompts long enough for every path of the expert products (few rows, lists, the library), in one batch with others."""
    cfg = O.config([O.parallel_layer(heads=2, kv_heads=1, dim=16, vdim=16, size=300, mlp=O.moe(8, 4, 4, 2, 128)),
                    O.retention_layer(heads=2, dim=16, vdim=16, mlp=O.moe(8, 4, 2, 1, 256))], width=128)
    w = model(cfg, 21, dtype)
    eng = engine(tmp_path, cfg, w, dtype, block=64)
    ids = {u: tokens(cfg, n, u) for u, n in ((0, 700), (1, 40), (2, 5))}
    want = {u: Want(cfg, w, t, dtype) for u, t in ids.items()}
    for cuts in ([700, 40, 5], [200, 20, 1], [90, 1, 1], [30, 2, 2]):
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
    """Keys and values only where a layer attends, a state where it has one; pool sizes count both."""
    from deepspeedsyclsupport_amd.inference.kv_cache import BlockedKVCache
    cfg = small()
    eng = engine(tmp_path, cfg, O.random_model(cfg, 9), "float32")
    c = eng.model.cache
    assert c.k[1] is None and tuple(c.state[1]["state"].shape) == (4, 3, 24, 16) and set(c.state[1]) == {"state"}
    assert tuple(c.k[0].shape[1:]) == (2, 16, 16) and tuple(c.v[0].shape[1:]) == (2, 16, 24)
    assert tuple(c.state[2]["state"].shape) == (4, 2, 40, 8) and tuple(c.state[2]["norm"].shape) == (4, 2, 2, 8)
    assert tuple(c.state[2]["peak"].shape) == (4, 2) and all(t.dtype == torch.float32 for t in c.state[2].values())
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
    for lacking in ("l0.mix.left.q.b", "l2.mix.right.norm", "l0.mlp.e3.up", "l4.mlp.router"):
        with pytest.raises(RuntimeError, match="not fully initialized"):
            engine(tmp_path, cfg, {k: v for k, v in w.items() if k != lacking}, "float32")
    for extra in ("l1.norm2", "l1.mlp.router", "head", "l0.mix.q"):
        with pytest.raises(ValueError, match="Cannot find container"):
            engine(tmp_path, cfg, {**w, extra: torch.zeros(64)}, "float32")
    for name, t in (("l0.mix.left.q.norm", torch.zeros(7)), ("l2.mix.right.i.b", torch.zeros(9)), ("l0.mlp.router", torch.zeros(7, 64))):
        with pytest.raises(ValueError, match="by the configuration"):
            engine(tmp_path, cfg, {**w, name: t}, "float32")
    for change in (lambda c: c["layers"][0].update(type="something else"), lambda c: c["layers"][0]["mlp"].update(kind="dense")):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        with pytest.raises(NotImplementedError):
            engine(tmp_path, bad, w, "float32")
    for path, value in ((("layers", 0, "mixer", "left", "kv_heads"), 4), (("layers", 1, "mixer", "decay"), [0.5]),
                        (("layers", 0, "mixer", "left", "rot", "dims"), 18), (("layers", 0, "mlp", "router", "groups", "count"), 4),
                        (("layers", 0, "mlp", "router", "top"), 5)):
        bad = json.loads(json.dumps(cfg))
        at = bad
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        with pytest.raises(ValueError):
            engine(tmp_path, bad, w, "float32")


def test_mixers_alone(tmp_path):
    """The two sides are mixers in their own right: a layer of one equals the parallel layer with the other one silenced."""
    from deepspeedsyclsupport_amd.inference.model_implementations.hybrid import DSHybridModel
    from deepspeedsyclsupport_amd.inference.model_implementations.transformer import DSModelSpec
    from deepspeedsyclsupport_amd.inference.v2 import AllocationMode, InferenceEngineV2, RaggedInferenceEngineConfig
    from deepspeedsyclsupport_amd.inference.v2.model_implementations.hybrid_archs import _MIXER_TENSORS
    pl = O.parallel_layer(left_scale=1.0, right_scale=1.0)
    ids = tokens({"vocab": 97}, 40)
    for side, kind, silent in (("left", "rotary_attention", "right_scale"), ("right", "matrix_memory", "left_scale")):
        cfg = O.config([json.loads(json.dumps(pl))])
        w = O.random_model(cfg, 14)
        cfg["layers"][0]["mixer"][silent] = 0.0
        spec = DSModelSpec(arch="test", vocab_size=97, hidden_size=64, num_layers=1, num_heads=4, num_kv_heads=2,
                           intermediate_size=0, norm="rms", pos="none", residual="pre_norm", embed_scale=1.7,
                           layer_specs=({"type": kind, "mixer": pl["mixer"][side], "mlp": None}, ))
        m = DSHybridModel(spec, dtype=torch.float32, device=torch.device("cpu"))
        lw = {key: w[f"l0.mix.{side}.{n}"] for n, key in _MIXER_TENSORS[kind].items()}
        with torch.no_grad():
            for name, t in m.shard_layer(0, {**lw, "norm1_w": w["l0.norm1"]}).items():
                m.layers[0].get_parameter(name).copy_(t)
            m.embed.copy_(w["embed"])
            m.lm_head.copy_(w["embed"])
            m.norm_w.copy_(w["final.norm"])
        eng = InferenceEngineV2(m, RaggedInferenceEngineConfig(
            state_manager={"memory_config": {"mode": AllocationMode.ALLOCATE, "size": 8}, "max_tracked_sequences": 2,
                           "max_ragged_sequence_count": 2, "max_context": 128}, kv_cache={"block_size": 16}))
        assert err(feed(eng, 0, ids, [30, 1]), O.forward(cfg, w, ids)) < 2e-4


@GPU
def test_weight_only_int8(tmp_path):
    """The framework's weight-only quantisation reaches these layers' projections too."""
    cfg = O.config([O.parallel_layer(heads=4, kv_heads=2, dim=64, vdim=64, r_heads=2, r_dim=63, r_vdim=64, mlp=O.moe(ff=64)),
                    O.retention_layer(heads=2, dim=64, vdim=64)], width=256, vocab=128)
    w = model(cfg, 12, "bfloat16")
    eng = engine(tmp_path, cfg, w, "bfloat16")
    ids = tokens(cfg, 40)
    want = O.forward(cfg, w, ids)
    eng.model.quantize_weights(8)
    assert err(feed(eng, 0, ids, [30, 1]), want) < 0.2 * want.std()


def _tp_run(path, ids, want, split):
    from deepspeedsyclsupport_amd.inference.v2 import (AllocationMode, RaggedInferenceEngineConfig, build_hf_engine)
    torch.set_num_threads(1)
    conf = RaggedInferenceEngineConfig(
        state_manager={"memory_config": {"mode": AllocationMode.ALLOCATE, "size": 16}, "max_tracked_sequences": 2,
                       "max_ragged_sequence_count": 2, "max_context": 256}, kv_cache={"block_size": 16},
        tensor_parallel={"tp_size": 2})
    eng = build_hf_engine(path, conf, dtype=torch.float32)
    mixers = [la.mixer for la in eng.model.layers]
    assert [m.parts[1].split if hasattr(m, "parts") else m.split for m in mixers] == split
    got = torch.cat([eng.put([0], [ids[:40]], logit_positions=[range(40)]),
                     eng.put([0], [ids[40:]], logit_positions=[range(10)])])
    assert err(got, want) < 5e-5


@pytest.mark.skipif(torch.cuda.is_available(), reason="ranks exchange host tensors")
def test_tensor_parallel(tmp_path):
    """Heads, states, experts and vocabulary over two ranks; attention whose norms span all heads, and head counts that do not
    divide, run whole on each."""
    cfg = O.config([O.parallel_layer(heads=6, kv_heads=2, r_heads=4, mlp=O.moe(ff=24)), O.parallel_layer(r_heads=3),
                    O.retention_layer(heads=4, mlp=O.moe(5, 2, 1, 1, 16)), O.retention_layer(heads=3)])
    w = O.random_model(cfg, 15)
    ids = tokens(cfg, 50)
    run_distributed(_tp_run, 2, save(tmp_path / "m", cfg, w), ids, O.forward(cfg, w, ids), [True, False, True, False])


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
