"""Perelorn through the framework: policy, weight loading, cache and state slots, ragged batches, scheduler, kernels —
against the plain implementation in `perelorn_oracle.py`."""
import json

import pytest
import torch

from ...common import run_distributed
from . import perelorn_oracle as O
from .test_vopepel import GPU, _one_thread, engine, err, feed, save, tokens  # noqa: F401

DTYPES = [pytest.param("float32", id="fp32"), pytest.param("float32", id="fp32-gpu", marks=GPU),
          pytest.param("bfloat16", id="bf16-gpu", marks=GPU)]


class Want:
    """The oracle's logits of one sequence and, per position, how far rounding the projections to bf16 moves them: the norms
    on sublayer outputs make some positions many times as sensitive as others."""

    def __init__(self, cfg, w, ids):
        self.logits = O.forward(cfg, w, ids)
        with O.Rounded():
            self.noise = self._dist(O.forward(cfg, w, ids), self.logits)

    @staticmethod
    def _dist(a, b):
        d = a.double().cpu() - b
        return (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt()

    def accepts(self, got, dtype, first=0, tol=2e-5):
        e = self._dist(got, self.logits[first:first + len(got)])
        if dtype == "float32":
            return e.max().item() < max(tol, 2e-3 * self.noise.max())   # (the two formats are 2^-15 apart)
        return e.max() < 4 * self.noise.max() and (len(e) < 30 or e.mean() < 2 * self.noise.mean())

    def shows(self, other):
        """A fault that moves the logits to `other` would not be taken for rounding."""
        d = self._dist(other, self.logits).max()
        assert d > 8 * self.noise.max(), (d, self.noise.max())
        return True


def small(**kw):
    """Unequal layers: every mixer with other sizes, with and without a feed-forward, norm parts that cut through heads."""
    return O.config([
        O.mamba2_layer(heads=6, groups=2, state=16, vdim=24, conv=3, norm_groups=4),
        O.latent_layer(heads=5, dim=16, rot_dim=8, vdim=24, kv_rank=40, q_rank=32, scale=0.23),
        O.lightning_layer(heads=3, dim=24, vdim=16, ff=40),
        O.latent_layer(heads=2, dim=24, rot_dim=16, vdim=8, kv_rank=64, q_rank=24, base=30.0, scale=0.4, ff=0),
        O.mamba2_layer(heads=3, groups=1, state=40, vdim=16, conv=5, norm_groups=1, ff=48),
        O.lightning_layer(heads=2, dim=16, vdim=40, decay=[1.0, 0.05]),
    ], **kw)


# ------------------------------------------------------------------------------------------------ whole model
@pytest.mark.parametrize("dtype", DTYPES)
def test_prompt_and_portions(tmp_path, dtype):
    """Whole prompts, token by token, and portions of several sizes (two tokens, odd ones, across page and state-chunk edges,
    on both sides of where attention and recurrences change kernels) give the oracle's logits at every position."""
    cfg = small()
    w = O.random_model(cfg, 1)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 150)
    want = Want(cfg, w, ids)
    for uid, cuts in enumerate(([150], [1], [2], [17, 3], [64, 64, 2, 1], [65, 1], [5, 129, 1], [16], [33], [66, 84])):
        assert want.accepts(feed(eng, uid, ids, cuts), dtype), cuts
        eng.flush(uid)


@pytest.mark.parametrize("dtype", DTYPES)
def test_residual_layer_by_layer(tmp_path, dtype):
    cfg = small()
    w = O.random_model(cfg, 2)
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
    w = O.random_model(cfg, 3)
    eng = engine(tmp_path, cfg, w, dtype, block=8, blocks=60, live=3)
    lens = {0: 90, 1: 41, 2: 7, 3: 180, 4: 66, 5: 1, 6: 75}
    ids = {u: tokens(cfg, n, u) for u, n in lens.items()}
    want = {u: Want(cfg, w, t) for u, t in ids.items()}
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
            assert want[u].accepts(got[row:row + cut[u]], dtype, at[u]), (step, u, at[u], cut[u])
            row, at[u] = row + cut[u], at[u] + cut[u]
            if at[u] == lens[u]:
                eng.flush(u)
                live.remove(u)
        step += 1
    assert eng._state_manager.free_blocks == 60 and eng._state_manager.free_slots == 3


@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens(tmp_path, dtype):
    """Sequences of one, two, three tokens: nothing before the start, in slots whose last owner left state and windows."""
    cfg = small(eps=1e-2, logit_scale=0.3)
    w = O.random_model(cfg, 4)
    eng = engine(tmp_path, cfg, w, dtype, live=2)
    for n in (70, 1, 2, 3, 5):
        ids = tokens(cfg, n, n)
        want = Want(cfg, w, ids)
        for cuts in ([n], [1]):
            assert want.accepts(feed(eng, 0, ids, cuts), dtype), (n, cuts)
            eng.flush(0)


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_key_and_sink(tmp_path, dtype):
    """A single key hundreds of tokens back that dominates its query, seen from a prompt, a portion and decoding, over two
    heads of which one's sink takes most of the weight and one's takes none."""
    cfg = O.config([O.latent_layer(heads=2, dim=32, rot_dim=8, vdim=32, kv_rank=96, q_rank=96, scale=0.5, base=1e6, ff=0)],
                   vocab=300, width=96)
    w = O.random_model(cfg, 5)
    # token 10 + i asks for token i and not for itself: its embedding is token i's turned by one place, and so is the map of
    # the query latent; from the latents on, queries and keys are the same maps
    w["embed"][10:20] = w["embed"][:10].roll(1, -1)
    w["l0.mix.dq"], w["l0.mix.dq.norm"] = w["l0.mix.dkv"][:96].roll(1, -1), w["l0.mix.dkv.norm"].clone()
    for h in range(2):
        w["l0.mix.uk"][h * 32:(h + 1) * 32] = w["l0.mix.uq"][h * 40:h * 40 + 32]
        w["l0.mix.uq"][h * 40 + 32:(h + 1) * 40] = 0       # no position: the score depends on the tokens alone
    w["l0.mix.sink"] = torch.tensor([14.0, -40.0]).bfloat16()
    eng = engine(tmp_path, cfg, w, dtype, blocks=120)
    ids = torch.cat([torch.arange(10), 20 + tokens(cfg, 579) % 280, torch.arange(10, 17)])
    want = Want(cfg, w, ids)
    other = want.logits.clone()                                # the far keys show, and so does the sink
    other[-7:] = O.forward(cfg, w, torch.cat([ids[300:310], ids[10:]]))[-7:]
    assert want.shows(other)
    assert want.shows(O.forward(cfg, {**w, "l0.mix.sink": torch.full((2, ), -40.0)}, ids))
    for uid, cuts in enumerate(([596], [560, 1], [301, 2], [500, 70, 26])):
        assert want.accepts(feed(eng, uid, ids, cuts), dtype), cuts
        eng.flush(uid)


@pytest.mark.parametrize("dtype", DTYPES)
def test_rotation(tmp_path, dtype):
    """A model whose scores are all rotation: positions that are one off would show, in prompts and decoding."""
    cfg = O.config([O.latent_layer(heads=3, dim=8, rot_dim=32, vdim=16, kv_rank=24, q_rank=16, scale=0.6, base=200.0, ff=0)])
    w = O.random_model(cfg, 6)
    for h in range(3):
        w["l0.mix.uq"][h * 40:h * 40 + 8] = 0
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 140)
    want = Want(cfg, w, ids)
    for uid, cuts in enumerate(([140], [30, 1], [100, 15, 2])):
        assert want.accepts(feed(eng, uid, ids, cuts), dtype), cuts


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_state(tmp_path, dtype):
    """Slow decays: tokens far back stay in the state; long decoding after a long prompt."""
    cfg = O.config([O.mamba2_layer(heads=4, groups=2, state=24, vdim=40, conv=4), O.lightning_layer(
        heads=2, dim=24, vdim=8, decay=[0.9999, 0.97]), O.mamba2_layer(heads=3, groups=3, state=72, vdim=8, conv=1,
                                                                       norm_groups=3, ff=32)], eps=5e-2)
    # (the wide eps keeps near-zero read-outs from being blown up by the norm behind them)
    w = O.random_model(cfg, 7)
    w["l0.mix.A_log"] -= 5
    w["l2.mix.dt_bias"] += 3   # strong decays next to slow ones
    w["embed"][:20] *= 6       # loud tokens at the start
    eng = engine(tmp_path, cfg, w, dtype)
    ids = torch.cat([tokens(cfg, 40) % 20, 20 + tokens(cfg, 290, 1) % 77])
    want = Want(cfg, w, ids)
    other = want.logits.clone()                                # the first tokens show at the end
    other[-50:] = O.forward(cfg, w, torch.cat([(ids[:40] + 1) % 20, ids[40:]]))[-50:]
    assert want.shows(other)
    for uid, cuts in enumerate(([330], [200, 1], [100, 17, 16, 2])):
        assert want.accepts(feed(eng, uid, ids, cuts), dtype), cuts


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,vocab,side", [(200, 131, 16), (132, 61, 3), (37, 50, 7)])
def test_model_widths(tmp_path, dtype, width, vocab, side):
    """Widths no vector or matrix tile divides."""
    cfg = O.config([O.latent_layer(heads=3, dim=20, rot_dim=6, vdim=12, kv_rank=27, q_rank=15, ff=45),
                    O.mamba2_layer(heads=3, groups=3, state=18, vdim=10, conv=2, norm_groups=5, ff=24),
                    O.lightning_layer(heads=2, dim=9, vdim=5)], width=width, vocab=vocab, side=side, eps=1e-3)
    w = O.random_model(cfg, 16)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 90)
    want = Want(cfg, w, ids)
    for u, cuts in enumerate(([90], [40, 2], [60, 1])):
        assert want.accepts(feed(eng, u, ids, cuts), dtype, tol=4e-5), cuts


@GPU
@pytest.mark.parametrize("latent", [(8, 128, 64, 128, 512, 384), (40, 64, 32, 64, 256, 128), (3, 192, 64, 256, 512, 64),
                                    (6, 30, 10, 20, 50, 40), (16, 64, 64, 96, 320, 200)])
@pytest.mark.parametrize("scan", [(8, 2, 128, 64, 8), (4, 1, 256, 128, 1), (6, 3, 64, 96, 3)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sizes(tmp_path, latent, scan, dtype):
    """Head sizes of real models and odd ones."""
    H, d, r, e, R, Q = latent
    h, g, n, v, parts = scan
    cfg = O.config([O.mamba2_layer(heads=h, groups=g, state=n, vdim=v, norm_groups=parts),
                    O.latent_layer(heads=H, dim=d, rot_dim=r, vdim=e, kv_rank=R, q_rank=Q),
                    O.lightning_layer(heads=g, dim=n // 2, vdim=v, ff=264)], width=256, vocab=130, side=32)
    w = O.random_model(cfg, 8)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 140)
    want = Want(cfg, w, ids)
    for u, cuts in enumerate(([140], [130, 1], [70, 5])):
        assert want.accepts(feed(eng, u, ids, cuts), dtype), cuts


# ------------------------------------------------------------------------------------------------ entry points
@pytest.mark.parametrize("dtype", [pytest.param("float32"), pytest.param("bfloat16", marks=GPU)])
def test_greedy_generation(tmp_path, dtype):
    """Continuous batching through `generate`: more requests than slots, a token budget that splits prompts. The oracle is
    followed along the engine's own tokens and the chosen token must be within rounding of its best."""
    cfg = small()
    w = O.random_model(cfg, 9)
    eng = engine(tmp_path, cfg, w, dtype, live=3)
    prompts = [tokens(cfg, n, 20 + n).tolist() for n in (5, 33, 1, 60, 18)]
    outs = eng.generate(prompts, max_new_tokens=9, token_budget=24)
    for p, o in zip(prompts, outs):
        assert len(o) == 9
        lg = O.forward(cfg, w, p + o[:-1])[len(p) - 1:]
        for row, tok in zip(lg, o):
            assert row.max() - row[tok] <= (1e-4 if dtype == "float32" else 0.15)
    assert eng._state_manager.free_slots == 3 and not eng._state_manager.tracked_sequences
    again = eng.generate(prompts[:2], max_new_tokens=9, eos_token_id=outs[0][2])
    if dtype == "float32":
        assert again[0] == outs[0][:outs[0].index(outs[0][2]) + 1]
    a, b = (eng.generate(prompts[:2], max_new_tokens=5, do_sample=True, temperature=0.8, top_k=20, top_p=0.9, seed=3)
            for _ in range(2))
    assert a == b


def test_geometry_and_pools(tmp_path):
    """One latent row per token and layer, state only where a layer carries one; pool sizes count both."""
    from deepspeedsyclsupport_amd.inference.kv_cache import BlockedKVCache
    cfg = small()
    eng = engine(tmp_path, cfg, O.random_model(cfg, 9), "float32")
    c = eng.model.cache
    assert c.k[0] is None and c.state[1] is None
    assert tuple(c.k[1].shape[1:]) == (1, 16, 48) and c.v[1].numel() == 0
    assert tuple(c.state[0]["state"].shape) == (4, 6, 24, 16) and c.state[0]["state"].dtype == torch.float32
    assert tuple(c.state[0]["conv"].shape) == (4, 2, 6 * 24 + 2 * 2 * 16) and "conv" not in c.state[2]
    assert c.bytes() == 64 * BlockedKVCache.block_bytes(eng.model.kv_geometry(), 16, torch.float32) + \
        4 * BlockedKVCache.slot_bytes(eng.model.state_geometry())
    handle = c.offload([1, 3])
    before = c.k[1][[1, 3]].clone()
    c.k[1].zero_()
    c.restore(handle)
    assert torch.equal(c.k[1][[1, 3]], before)


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
    with pytest.raises(RuntimeError, match="not fully initialized"):
        engine(tmp_path, cfg, {k: v for k, v in w.items() if k != "l1.mix.sink"}, "float32")
    with pytest.raises(RuntimeError, match="not fully initialized"):
        engine(tmp_path, cfg, {k: v for k, v in w.items() if k != "side.embed"}, "float32")
    with pytest.raises(ValueError, match="Cannot find container"):
        engine(tmp_path, cfg, {**w, "l0.norm2": torch.zeros(64)}, "float32")     # that layer has no feed-forward
    for name, t in (("l0.mix.A_log", torch.zeros(7)), ("side.embed", torch.zeros(97, 5)), ("l2.mix.norm", torch.zeros(9))):
        with pytest.raises(ValueError, match="by the configuration"):
            engine(tmp_path, cfg, {**w, name: t}, "float32")
    for change in (lambda c: c["layers"][0].update(type="something else"), lambda c: c["layers"][1]["mlp"].update(kind="moe")):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        with pytest.raises(NotImplementedError):
            engine(tmp_path, bad, w, "float32")
    for i, key, value in ((0, "groups", 4), (0, "norm_groups", 7), (2, "decay", [0.5]), (1, "rot", {"base": 10.0, "dims": 10})):
        bad = json.loads(json.dumps(cfg))
        bad["layers"][i]["mixer"][key] = value
        with pytest.raises(ValueError):
            engine(tmp_path, bad, w, "float32")


@GPU
def test_weight_only_int8(tmp_path):
    """The framework's weight-only quantisation reaches these layers' projections too."""
    cfg = O.config([O.mamba2_layer(heads=4, groups=2, state=64, vdim=64, ff=256), O.lightning_layer(heads=2, dim=64, vdim=64),
                    O.latent_layer(heads=4, dim=64, rot_dim=32, vdim=64, kv_rank=128, q_rank=128, ff=256)], width=256,
                   vocab=128, side=64)
    w = O.random_model(cfg, 12)
    eng = engine(tmp_path, cfg, w, "bfloat16")
    ids = tokens(cfg, 40)
    want = O.forward(cfg, w, ids)
    eng.model.quantize_weights(8)
    assert err(feed(eng, 0, ids, [30, 1]), want) < 0.2


def _tp_run(path, ids, want, split):
    from deepspeedsyclsupport_amd.inference.v2 import (AllocationMode, RaggedInferenceEngineConfig, build_hf_engine)
    torch.set_num_threads(1)
    conf = RaggedInferenceEngineConfig(
        state_manager={"memory_config": {"mode": AllocationMode.ALLOCATE, "size": 16}, "max_tracked_sequences": 2,
                       "max_ragged_sequence_count": 2, "max_context": 256}, kv_cache={"block_size": 16},
        tensor_parallel={"tp_size": 2})
    eng = build_hf_engine(path, conf, dtype=torch.float32)
    assert [la.mixer.split for la in eng.model.layers if la.mixer.kind == "mamba2"] == split
    got = torch.cat([eng.put([0], [ids[:40]], logit_positions=[range(40)]),
                     eng.put([0], [ids[40:]], logit_positions=[range(10)])])
    assert err(got, want) < 2e-5


@pytest.mark.skipif(torch.cuda.is_available(), reason="ranks exchange host tensors")
def test_tensor_parallel(tmp_path):
    """Heads, groups, states, windows, feed-forward and vocabulary over two ranks; mixers whose norm spans all heads run whole
    on each."""
    cfg = O.config([O.mamba2_layer(heads=6, groups=2, state=16, vdim=24, conv=3, norm_groups=2, ff=40),
                    O.mamba2_layer(heads=4, groups=2, state=16, vdim=24, norm_groups=1),
                    O.latent_layer(heads=4), O.lightning_layer(heads=3, vdim=16)])
    w = O.random_model(cfg, 15)
    ids = tokens(cfg, 50)
    run_distributed(_tp_run, 2, save(tmp_path / "m", cfg, w), ids, O.forward(cfg, w, ids), [True, False])


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

    assert err(read(0), la[[3, 39]]) < 2e-5
    assert err(read(1), torch.stack([lb[1], lb[89], la[40]])) < 2e-5
    assert eng._state_manager.free_blocks == 3 and eng._state_manager.free_slots == 4
