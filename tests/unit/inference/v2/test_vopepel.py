"""Vopepel through the framework: policy, weight loading, cache and state slots, ragged batches, scheduler, kernels —
against the plain implementation in `vopepel_oracle.py`."""
import json

import pytest
import torch

from ...common import run_distributed
from . import vopepel_oracle as O

GPU = pytest.mark.gpu
# dtype name, tolerance of the logits (rms over the vocabulary; the logits have unit scale)
PRECISION = [pytest.param("float32", 2e-5, id="fp32"), pytest.param("float32", 2e-5, id="fp32-gpu", marks=GPU),
             pytest.param("bfloat16", 4e-2, id="bf16-gpu", marks=GPU)]
ON_GPU = [pytest.param(torch.float32, marks=GPU), pytest.param(torch.bfloat16, marks=GPU)]


@pytest.fixture(autouse=True)
def _one_thread():
    """The host versions are many tiny ops: threads only slow them down."""
    n = torch.get_num_threads()
    torch.set_num_threads(1)
    yield
    torch.set_num_threads(n)


def small(streams=3):
    """Unequal layers: other widths, ratios, chunk sizes and clamps in every one, one without a feed-forward."""
    return O.config([
        O.delta_layer(heads=6, kv_heads=2, dim=16, vdim=24, conv=3),
        O.attention_layer(heads=6, kv_heads=2, dim=32, vdim=16, size=24, scale=0.21),
        O.attention_layer(heads=3, kv_heads=3, dim=24, vdim=40, size=70, scale=0.35, softcap=4.0, v_mix=False, ff=0),
        O.attention_layer(heads=4, kv_heads=2, dim=40, vdim=16, size=1, v_mix=True, ff=40, limit=0.3),
        O.delta_layer(heads=2, kv_heads=2, dim=40, vdim=16, conv=5, ff=0),
        O.attention_layer(heads=2, kv_heads=2, dim=16, vdim=16, size=33, v_mix=True, limit=2.5),
    ], streams=streams)


def save(tmp_path, cfg, weights):
    from safetensors.torch import save_file
    tmp_path.mkdir(exist_ok=True)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in weights.items()}, str(tmp_path / "model.safetensors"))
    return str(tmp_path)


def engine(tmp_path, cfg, weights, dtype, block=16, blocks=64, live=4, **state):
    from deepspeedsyclsupport_amd.inference.v2 import (AllocationMode, RaggedInferenceEngineConfig, build_hf_engine)
    conf = RaggedInferenceEngineConfig(
        state_manager={"memory_config": {"mode": AllocationMode.ALLOCATE, "size": blocks}, "max_tracked_sequences": live,
                       "max_ragged_sequence_count": live, "max_ragged_batch_size": 2048, "max_context": block * blocks,
                       **state}, kv_cache={"block_size": block})
    return build_hf_engine(save(tmp_path / "m", cfg, weights), conf, dtype=getattr(torch, dtype))


def err(got, want):
    d = got.double().cpu() - want.double()
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt().max().item()


def tokens(cfg, n, seed=0):
    return torch.randint(0, cfg["vocab"], (n, ), generator=torch.Generator().manual_seed(seed))


def feed(eng, uid, toks, cuts):
    """All logits of one sequence fed in portions of the given sizes (the last one repeats)."""
    out, at, i = [], 0, 0
    while at < toks.numel():
        n = min(cuts[min(i, len(cuts) - 1)], toks.numel() - at)
        out.append(eng.put([uid], [toks[at:at + n]], logit_positions=[list(range(n))]).float().cpu())
        at, i = at + n, i + 1
    return torch.cat(out)


# ------------------------------------------------------------------------------------------------ whole model
@pytest.mark.parametrize("dtype,tol", PRECISION)
@pytest.mark.parametrize("streams", [3, 1])
def test_prompt_and_portions(tmp_path, dtype, tol, streams):
    """Whole prompts, token by token, and portions of several sizes (two tokens, odd ones, across page, mask-chunk and
    state-chunk edges) give the oracle's logits at every position."""
    cfg = small(streams)
    w = O.random_model(cfg, 1)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 150)
    want = O.forward(cfg, w, ids)
    for uid, cuts in enumerate(([150], [1], [2], [17, 3], [64, 64, 2, 1], [65, 1], [5, 129, 1], [16], [33])):
        assert err(feed(eng, uid, ids, cuts), want) < tol, cuts
        eng.flush(uid)


@pytest.mark.parametrize("dtype,tol", PRECISION)
def test_residual_stream_layer_by_layer(tmp_path, dtype, tol):
    cfg = small()
    w = O.random_model(cfg, 2)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 30)
    trace, want = [], []
    O.forward(cfg, w, ids, trace=want)
    seq = eng._state_manager.get_or_create_sequence(0)
    eng._state_manager.allocate_blocks(seq, 30)
    eng._batch.clear()
    eng._batch.insert_sequence(seq, ids)
    eng._batch.finalize()
    eng.model.forward_ragged(eng._batch.input_ids(), eng._batch.meta, trace=trace)
    assert len(trace) == len(want)
    for a, b in zip(trace, want):
        assert (a.double().cpu() - b).abs().max() < 8 * tol * max(1.0, b.abs().max().item())


@pytest.mark.parametrize("dtype,tol", PRECISION)
def test_mixed_batches_and_reuse(tmp_path, dtype, tol):
    """Unequal requests in one batch (portions beside single tokens, one pausing, one joining late), then new requests on
    the freed pages and slots: each equals itself alone."""
    cfg = small()
    w = O.random_model(cfg, 3)
    eng = engine(tmp_path, cfg, w, dtype, block=8, blocks=40, live=3)
    lens = {0: 90, 1: 41, 2: 7, 3: 100, 4: 66, 5: 1, 6: 75}
    ids = {u: tokens(cfg, n, u) for u, n in lens.items()}
    want = {u: O.forward(cfg, w, t) for u, t in ids.items()}
    at = {u: 0 for u in lens}
    waiting, live, step = list(lens), [], 0
    g = torch.Generator().manual_seed(0)
    sizes = [1, 2, 3, 16, 17, 40, 1, 1]
    while waiting or live:
        while waiting and len(live) < 3:
            live.append(waiting.pop(0))
        batch = [u for u in live if torch.rand(1, generator=g) < 0.8] or live[:1]
        cut = {u: min(sizes[int(torch.randint(0, 8, (1, ), generator=g))], lens[u] - at[u]) for u in batch}
        got = eng.put(batch, [ids[u][at[u]:at[u] + cut[u]] for u in batch],
                      logit_positions=[range(cut[u]) for u in batch]).float().cpu()
        row = 0
        for u in batch:
            assert err(got[row:row + cut[u]], want[u][at[u]:at[u] + cut[u]]) < tol, (step, u, at[u], cut[u])
            row, at[u] = row + cut[u], at[u] + cut[u]
            if at[u] == lens[u]:
                eng.flush(u)
                live.remove(u)
        step += 1
    assert eng._state_manager.free_blocks == 40 and eng._state_manager.free_slots == 3


@pytest.mark.parametrize("dtype,tol", PRECISION)
@pytest.mark.parametrize("size", [1, 15, 16, 50, 129])
def test_chunk_edges(tmp_path, dtype, tol, size):
    """One attention layer with sharp scores: keys just inside and just outside a chunk, at page borders, in prompts and
    decoded."""
    cfg = O.config([O.attention_layer(heads=2, kv_heads=1, dim=32, vdim=32, size=size, scale=1.0, softcap=20.0, ff=0)],
                   streams=2)
    w = O.random_model(cfg, 4, peak=1.6)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 140)
    want = O.forward(cfg, w, ids)
    wrong = O.forward({**cfg, "layers": [{**cfg["layers"][0], "mixer": {**cfg["layers"][0]["mixer"],
                                                                        "mask": {"size": size + 1}}}]}, w, ids)
    assert err(wrong, want) > (5 if size < 129 else 1) * tol  # an edge that is one off would show
    assert err(feed(eng, 0, ids, [140]), want) < tol
    assert err(feed(eng, 1, ids, [30, 1]), want) < tol


@pytest.mark.parametrize("dtype,tol", PRECISION)
def test_far_key_and_score_cap(tmp_path, dtype, tol):
    """A single key hundreds of tokens back that dominates its query, seen from a prompt and from decoding."""
    cfg = O.config([O.attention_layer(heads=4, kv_heads=2, dim=64, vdim=32, size=700, scale=1.0, softcap=12.0,
                                      ff=0)], vocab=300, width=96, streams=2)
    w = O.random_model(cfg, 5, peak=1.0)
    w["l0.mix.k"][:64] = w["l0.mix.q"][:64]  # a token's key answers the query of the same token
    eng = engine(tmp_path, cfg, w, dtype, blocks=120)
    ids = torch.cat([torch.arange(300), torch.arange(299, -1, -1)])[:596]
    want = O.forward(cfg, w, ids)
    assert err(feed(eng, 0, ids, [596]), want) < tol
    assert err(feed(eng, 1, ids, [560, 1]), want) < tol
    eng.flush(0)
    assert err(feed(eng, 2, ids, [301, 2]), want) < tol


@pytest.mark.parametrize("dtype,tol", PRECISION)
@pytest.mark.parametrize("softcap", [None, 1.5, 33.0, 34.0, 90.0])
def test_score_caps(tmp_path, dtype, tol, softcap):
    """No cap, one that bends most scores, and ones on both sides of where the prefill kernel stops taking the cap for
    the maximum; no chunks; values not mixed; sharp scores."""
    cfg = O.config([O.attention_layer(heads=4, kv_heads=1, dim=48, vdim=72, size=10**6, scale=0.5, softcap=softcap,
                                      v_mix=False, ff=0)], streams=2)
    del cfg["layers"][0]["mixer"]["v_mix"]
    if softcap is None:
        del cfg["layers"][0]["mixer"]["softcap"], cfg["layers"][0]["mixer"]["mask"]
    w = O.random_model(cfg, 14, peak=1.6)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 150)
    want = O.forward(cfg, w, ids)
    assert err(feed(eng, 0, ids, [150]), want) < tol
    assert err(feed(eng, 1, ids, [120, 1]), want) < tol


@pytest.mark.parametrize("dtype,tol", PRECISION)
def test_long_state(tmp_path, dtype, tol):
    """Slow decays: tokens far back stay in the state; long decoding after a long prompt."""
    cfg = O.config([O.delta_layer(heads=4, kv_heads=2, dim=24, vdim=40, conv=4, ff=0),
                    O.delta_layer(heads=3, kv_heads=1, dim=72, vdim=8, conv=1, ff=32)], streams=2)
    w = O.random_model(cfg, 6)
    w["l0.mix.A_log"] -= 4
    w["l1.mix.dt_bias"] += 3   # strong decays next to slow ones
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 330)
    want = O.forward(cfg, w, ids)
    assert err(feed(eng, 0, ids, [330]), want) < tol
    assert err(feed(eng, 1, ids, [200, 1]), want) < tol
    assert err(feed(eng, 2, ids, [100, 17, 16, 2]), want) < tol


@pytest.mark.parametrize("dtype,tol", PRECISION)
@pytest.mark.parametrize("width,vocab,streams", [(200, 131, 2), (132, 61, 8), (37, 50, 5)])
def test_model_widths(tmp_path, dtype, tol, width, vocab, streams):
    """Widths no vector or matrix tile divides, other stream counts, a feed-forward of 1-wide remainder."""
    cfg = O.config([O.attention_layer(heads=3, kv_heads=1, dim=20, vdim=12, size=31, ff=45),
                    O.delta_layer(heads=3, kv_heads=3, dim=18, vdim=10, conv=2, ff=24),
                    O.attention_layer(heads=2, kv_heads=1, dim=16, vdim=12, size=20, ff=0)], width=width, vocab=vocab,
                   streams=streams, residual_mult=1.0, eps=1e-3)
    w = O.random_model(cfg, 16)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 90)
    want = O.forward(cfg, w, ids)
    for u, cuts in enumerate(([90], [40, 2], [60, 1])):
        assert err(feed(eng, u, ids, cuts), want) < 2 * tol, cuts


@GPU
@pytest.mark.parametrize("dims", [(8, 4, 128, 128, 128, 128), (4, 2, 256, 256, 256, 192), (4, 4, 64, 96, 80, 64),
                                  (12, 1, 48, 20, 72, 200), (2, 1, 20, 33, 36, 28)])
@pytest.mark.parametrize("dtype,tol", [("float32", 3e-5), ("bfloat16", 4e-2)])
def test_sizes(tmp_path, dims, dtype, tol):
    """Head sizes of real models and odd ones (GQA groups above 8, widths no tile divides)."""
    H, G, ddk, ddv, adk, adv = dims
    cfg = O.config([O.delta_layer(heads=H, kv_heads=G, dim=ddk, vdim=ddv), O.attention_layer(
        heads=H, kv_heads=G, dim=adk, vdim=adv, size=90, scale=adk**-0.5)], width=256, vocab=130, streams=4)
    w = O.random_model(cfg, 7)
    eng = engine(tmp_path, cfg, w, dtype)
    ids = tokens(cfg, 200)
    want = O.forward(cfg, w, ids, torch.float64)
    for u, cuts in enumerate(([200], [130, 1], [70, 5])):
        assert err(feed(eng, u, ids, cuts), want) < tol, cuts


# ------------------------------------------------------------------------------------------------ entry points
@pytest.mark.parametrize("dtype", [pytest.param("float32"), pytest.param("bfloat16", marks=GPU)])
def test_greedy_generation(tmp_path, dtype):
    """Continuous batching through `generate`: more requests than slots, a token budget that splits prompts. Compared
    with the oracle's greedy choice; with bf16, tokens whose margin is within rounding may differ, so the oracle is
    followed along the engine's own tokens and the chosen token must be close to its best."""
    cfg = small()
    w = O.random_model(cfg, 8)
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
    cut = outs[0].index(outs[0][2]) + 1
    if dtype == "float32":
        assert again[0] == outs[0][:cut]
    a = eng.generate(prompts[:2], max_new_tokens=5, do_sample=True, temperature=0.8, top_k=20, top_p=0.9, seed=3)
    b = eng.generate(prompts[:2], max_new_tokens=5, do_sample=True, temperature=0.8, top_k=20, top_p=0.9, seed=3)
    assert a == b


def test_scheduling_slots(tmp_path):
    from deepspeedsyclsupport_amd.inference.v2 import SchedulingResult
    cfg = small()
    eng = engine(tmp_path, cfg, O.random_model(cfg, 9), "float32", live=4, state_slots=2)
    assert eng._state_manager.free_slots == 2
    assert eng.can_schedule([1, 2], [4, 4]) == SchedulingResult.Success
    assert eng.can_schedule([1, 2, 3], [4, 4, 4]) == SchedulingResult.EngineSequenceLimitExceeded
    with pytest.raises(ValueError, match="outside the vocabulary"):
        eng.put([1], [torch.tensor([3, cfg["vocab"]])])
    eng.put([1, 2], [tokens(cfg, 4), tokens(cfg, 3)])
    assert eng.query(3, 8, 4) == (0, 0)
    eng.flush(1)
    assert eng.query(3, 8, 4)[0] == 8


def test_geometry_and_pools(tmp_path):
    """Caches only where a layer has keys and values, state only where it carries one; automatic pool sizes count both."""
    from deepspeedsyclsupport_amd.inference.kv_cache import BlockedKVCache
    cfg = small()
    eng = engine(tmp_path, cfg, O.random_model(cfg, 9), "float32")
    c = eng.model.cache
    assert c.k[0] is None and c.state[1] is None
    assert tuple(c.k[1].shape[1:]) == (2, 16, 32) and tuple(c.v[1].shape[1:]) == (2, 16, 16)
    assert tuple(c.state[0]["state"].shape) == (4, 6, 24, 16) and c.state[0]["state"].dtype == torch.float32
    per_block = BlockedKVCache.block_bytes(eng.model.kv_geometry(), 16, torch.float32)
    per_slot = BlockedKVCache.slot_bytes(eng.model.state_geometry())
    assert c.bytes() == 64 * per_block + 4 * per_slot
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
        engine(tmp_path, cfg, {k: v for k, v in w.items() if k != "l0.mix.b"}, "float32")
    with pytest.raises(ValueError, match="Cannot find container"):
        engine(tmp_path, cfg, {**w, "l0.mix.extra": torch.zeros(3)}, "float32")
    with pytest.raises(ValueError, match="by the configuration"):
        engine(tmp_path, cfg, {**w, "l0.mix.A_log": torch.zeros(7)}, "float32")
    bad = json.loads(json.dumps(cfg))
    bad["layers"][0]["type"] = "something else"
    with pytest.raises(NotImplementedError):
        engine(tmp_path, bad, w, "float32")


@GPU
def test_weight_only_int8(tmp_path):
    """The framework's weight-only quantisation reaches the hybrid layers' projections too."""
    cfg = O.config([O.delta_layer(heads=4, kv_heads=4, dim=32, vdim=64, ff=256),
                    O.attention_layer(heads=4, kv_heads=4, dim=64, vdim=64, size=64, scale=0.125, ff=256)], width=256,
                   vocab=128, streams=2)
    w = O.random_model(cfg, 12)
    eng = engine(tmp_path, cfg, w, "bfloat16")
    ids = tokens(cfg, 40)
    want = O.forward(cfg, w, ids)
    eng.model.quantize_weights(8)
    assert err(feed(eng, 0, ids, [30, 1]), want) < 0.12


def _tp_run(path, ids, want):
    from deepspeedsyclsupport_amd.inference.v2 import (AllocationMode, RaggedInferenceEngineConfig, build_hf_engine)
    torch.set_num_threads(1)
    conf = RaggedInferenceEngineConfig(
        state_manager={"memory_config": {"mode": AllocationMode.ALLOCATE, "size": 16}, "max_tracked_sequences": 2,
                       "max_ragged_sequence_count": 2, "max_context": 256}, kv_cache={"block_size": 16},
        tensor_parallel={"tp_size": 2})
    eng = build_hf_engine(path, conf, dtype=torch.float32)
    assert eng.model.layers[0].mixer.H == 3
    got = torch.cat([eng.put([0], [ids[:40]], logit_positions=[range(40)]),
                     eng.put([0], [ids[40:]], logit_positions=[range(10)])])
    assert err(got, want) < 2e-5


@pytest.mark.skipif(torch.cuda.is_available(), reason="ranks exchange host tensors")
def test_tensor_parallel(tmp_path):
    """Heads, states, convolution windows, feed-forward and vocabulary over two ranks."""
    cfg = O.config([O.delta_layer(heads=6, kv_heads=2, dim=16, vdim=24, conv=3),
                    O.attention_layer(heads=6, kv_heads=2, dim=32, vdim=16, size=24),
                    O.attention_layer(heads=4, kv_heads=2, dim=24, vdim=16, size=70, ff=0)])
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

    assert err(read(0), la[[3, 39]]) < 2e-5
    assert err(read(1), torch.stack([lb[1], lb[89], la[40]])) < 2e-5
    assert eng._state_manager.free_blocks == 3 and eng._state_manager.free_slots == 4
