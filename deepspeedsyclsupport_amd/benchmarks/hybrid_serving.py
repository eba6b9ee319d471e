"""Serving throughput of hybrid decoders beside the uniform Llama-style decoder at equal width, feed-forward, head and layer
counts, all through the ragged engine with random bf16 weights: whole-prompt prefill and batched decoding.

* hybrid: Vopepel layers (gated delta rule, chunked attention, residual streams)
* perelorn: Perelorn layers (Mamba-2, latent attention, lightning attention, norms on sublayer outputs, token-side input)
* lefisun: Lefisun layers (chunked rotary attention beside a matrix memory, retention, routed experts); beside it
  uniform_moe, the Llama-style decoder with the same experts (Mixtral's routing), and the others with a dense feed-forward as
  wide as the experts of a token together
* nigilorn: Nigilorn layers (selective state spaces, windowed attention, windowed latent attention, gated residual with norms on
  both sides, token-side input, one dense feed-forward, then plain routed experts beside a shared one)

    python bench.py --workload hybrid [--sizes 2048,4096] [--model-kind hybrid|perelorn|lefisun|nigilorn|uniform|uniform_moe|...]
"""
import json
import math
import time

import torch

SIZES = {2048: dict(ff=5632, heads=16, kv=8), 4096: dict(ff=14336, heads=32, kv=8)}
PATTERN = ("delta", "attention", "attention", "delta", "attention", "attention", "delta", "attention")
HEAD, CHUNK, STREAMS, VOCAB, SIDE = 128, 2048, 4, 32000, 256


# Perelorn: the delta layers' places go to Mamba-2 and lightning, attention to latent attention; every layer keeps its
# feed-forward, so that the projections are of one size
PERELORN = ("mamba2", "latent_attention", "lightning", "mamba2", "latent_attention", "lightning", "mamba2", "latent_attention")
KINDS = {"both": ("hybrid", "uniform"), "moe": ("lefisun", "uniform_moe"),
         "close": ("nigilorn", "perelorn", "lefisun"),   # the last design and those it shares most with
         "all": ("hybrid", "perelorn", "uniform", "lefisun", "uniform_moe", "nigilorn")}
# Lefisun: attention of the others' size beside a memory of half its heads, retention in the places of their recurrences
EXPERTS, TOP, GROUPS, KEEP = 32, 4, 4, 2
LEFISUN = ("parallel", "retention") * 4
# Nigilorn: state spaces in the places of the recurrences, the two kinds of attention by turns
NIGILORN = ("mamba1", "window_attention", "mamba1", "latent_attention") * 2


def specs(width):
    """{kind: model spec} of one size."""
    from ..inference.model_implementations.transformer import DSModelSpec
    s = SIZES[width]
    common = dict(vocab_size=VOCAB, hidden_size=width, num_layers=len(PATTERN), num_heads=s["heads"],
                  num_kv_heads=s["kv"], intermediate_size=s["ff"], head_dim=HEAD)
    mlp = {"kind": "dense", "ff": s["ff"], "limit": 7.0}
    mixers = {"delta": {"heads": s["heads"], "kv_heads": s["kv"], "dim": HEAD, "vdim": HEAD, "conv": 4},
              "attention": {"heads": s["heads"], "kv_heads": s["kv"], "dim": HEAD, "vdim": HEAD, "scale": HEAD**-0.5,
                            "softcap": 30.0, "mask": {"size": CHUNK}, "v_mix": True}}
    hybrid = DSModelSpec(arch="vopepel", norm="ln", norm_bias=False, pos="none", streams=STREAMS, residual_mult=0.7,
                         layer_specs=tuple({"type": t, "mixer": mixers[t], "mlp": mlp} for t in PATTERN), **common)
    uniform = DSModelSpec(arch="llama", norm="rms", pos="rope", max_positions=16384, **common)
    h = s["heads"]
    mixers = {"mamba2": {"heads": 2 * h, "groups": 1, "state": HEAD, "vdim": HEAD // 2, "conv": 4, "norm_groups": 1},
              "lightning": {"heads": h, "dim": HEAD, "vdim": HEAD, "decay": [math.exp(-2**(-8 * (i + 1) / h)) for i in range(h)]},
              "latent_attention": {"heads": h, "dim": HEAD, "rot_dim": 64, "vdim": HEAD, "kv_rank": 512, "q_rank": 1536,
                                   "rot": {"base": 10000.0, "dims": 64}, "scale": (HEAD + 64)**-0.5}}
    perelorn = DSModelSpec(arch="perelorn", norm="rms", pos="none", residual="post_norm", token_side=SIDE, logit_scale=1.0,
                           layer_specs=tuple({"type": t, "mixer": mixers[t], "mlp": {"kind": "gelu", "ff": s["ff"]}}
                                             for t in PERELORN), **common)
    ff = s["ff"] // TOP
    mixers = {"parallel": {"left": {"heads": h, "kv_heads": s["kv"], "dim": HEAD, "vdim": HEAD, "scale": HEAD**-0.5,
                                    "mask": {"size": CHUNK}, "rot": {"base": 5e5, "dims": HEAD // 2, "scaling": {"factor": 4.0}}},
                           "right": {"heads": h // 2, "dim": HEAD, "vdim": HEAD, "gate_cap": 15.0},
                           "left_scale": 0.8, "right_scale": 0.6},
              "retention": {"heads": h, "dim": HEAD, "vdim": HEAD, "rot": {"base": 1e4, "dims": HEAD},
                            "decay": [1 - 2**(-5 - 3 * i / h) for i in range(h)]}}
    mlp = {"kind": "routed", "expert": {"ff": ff}, "router": {"experts": EXPERTS, "top": TOP, "groups": {"count": GROUPS,
                                                                                                        "keep": KEEP}}}
    lefisun = DSModelSpec(arch="lefisun", norm="rms", pos="none", residual="pre_norm", tie_embeddings=True,
                          layer_specs=tuple({"type": t, "mixer": mixers[t], "mlp": mlp} for t in LEFISUN), **common)
    uniform_moe = DSModelSpec(arch="mixtral", norm="rms", pos="rope", max_positions=16384, num_experts=EXPERTS, moe_top_k=TOP,
                              **{**common, "intermediate_size": ff})
    yarn = {"type": "yarn", "factor": 4.0, "fast": 32.0, "slow": 1.0, "original": 4096}
    mixers = {"mamba1": {"inner": 2 * width, "state": 16, "dt_rank": width // 16, "conv": 4},
              "window_attention": {"heads": h, "kv_heads": s["kv"], "dim": HEAD, "vdim": HEAD, "scale": HEAD**-0.5,
                                   "mask": {"size": CHUNK}, "rot": {"base": 5e5, "dims": HEAD // 2, "pairs": "neighbours",
                                                                    "scaling": yarn}},
              "latent_attention": {"heads": h, "dim": HEAD, "rot_dim": 64, "vdim": HEAD, "kv_rank": 512, "sink": False,
                                   "mask": {"size": CHUNK}, "rot": {"base": 10000.0, "dims": 64, "pairs": "neighbours",
                                                                    "scaling": yarn}, "scale": (HEAD + 64)**-0.5}}
    mlp = {**mlp, "act": "relu2", "shared": {"ff": ff},
           "router": {"experts": EXPERTS, "top": TOP, "score": "sigmoid", "scale": 2.5,
                      "groups": {"count": GROUPS, "keep": KEEP, "best": 2}}}
    dense = {"kind": "silu_glu", "ff": s["ff"]}
    nigilorn = DSModelSpec(arch="nigilorn", norm="rms", pos="none", residual="sandwich", residual_gate=True, token_side=SIDE,
                           layer_specs=tuple({"type": t, "mixer": mixers[t], "mlp": mlp if i else dense}
                                             for i, t in enumerate(NIGILORN)), **common)
    return {"hybrid": hybrid, "perelorn": perelorn, "uniform": uniform, "lefisun": lefisun, "uniform_moe": uniform_moe,
            "nigilorn": nigilorn}


def build(spec, device, blocks):
    from ..inference.model_implementations.hybrid import model_class
    from ..inference.v2 import AllocationMode, InferenceEngineV2, RaggedInferenceEngineConfig
    from ..inference.v2.engine_factory import _apply_decode_layout
    torch.manual_seed(0)
    model = model_class(spec)(spec, dtype=torch.bfloat16, device=device)
    with torch.no_grad():
        for name, p in model.named_parameters():
            if name.endswith(".decay"):
                p.copy_(-p.normal_(0, 0.5).exp())   # rates of a selective state space
            elif p.dim() >= 2 and p.dtype == torch.bfloat16:
                p.normal_(0, 0.02)
            elif p.dim() == 2 and p.shape[0] == p.shape[1]:
                p.copy_(torch.eye(p.shape[0]))      # stream mixing
            elif p.dim() == 2:
                p.normal_(0, 0.3)                   # convolution taps
    _apply_decode_layout(model, "auto", 1, torch.device(device))
    cfg = RaggedInferenceEngineConfig(
        state_manager={"memory_config": {"mode": AllocationMode.ALLOCATE, "size": blocks}, "max_ragged_batch_size": 8192,
                       "max_ragged_sequence_count": 64, "max_tracked_sequences": 64, "max_context": 16384},
        kv_cache={"block_size": 64})
    return InferenceEngineV2(model, cfg)


def timed(fn, iters, warmup=2):
    for _ in range(warmup):
        fn()
    torch.cuda.synchronize()
    t = time.perf_counter()
    for _ in range(iters):
        fn()
    torch.cuda.synchronize()
    return (time.perf_counter() - t) / iters


def measure(spec, device, prompts, batches, context, iters, log):
    eng = build(spec, device, blocks=64 * (context // 64 + 2) + 256)
    g = torch.Generator().manual_seed(0)
    out = {"prefill_tok_s": {}, "decode_tok_s": {}, "decode_ms": {}}
    for n, length in prompts:
        toks = [torch.randint(0, spec.vocab_size, (length, ), generator=g) for _ in range(n)]

        def prefill():
            eng.put(list(range(n)), toks)
            for u in range(n):
                eng.flush(u)

        t = timed(prefill, iters)
        out["prefill_tok_s"][f"{n}x{length}"] = round(n * length / t, 1)
        log(f"[bench] {spec.arch} w{spec.hidden_size} prefill {n}x{length}: {t * 1e3:.2f} ms")
    for u in range(max(batches)):
        logits = eng.put([u], [torch.randint(0, spec.vocab_size, (context, ), generator=g)])
    if not torch.isfinite(logits.float()).all():
        raise RuntimeError(f"{spec.arch}: logits are not finite")
    for b in batches:
        one = [torch.tensor([u % spec.vocab_size]) for u in range(b)]
        t = timed(lambda: eng.put(list(range(b)), one), iters * 2)
        out["decode_tok_s"][str(b)] = round(b / t, 1)
        out["decode_ms"][str(b)] = round(t * 1e3, 3)
        log(f"[bench] {spec.arch} w{spec.hidden_size} decode b{b} ctx{context}: {t * 1e3:.3f} ms")
    return out


def run(sizes=(2048, 4096), kind="both", iters=10, prompts=((1, 8192), (4, 2048), (16, 128)), batches=(1, 16, 64),
        context=1536, log=print):
    device = torch.device("cuda", torch.cuda.current_device())
    rows = []
    for width in sizes:
        row = {"width": width, "layers": len(PATTERN), **SIZES[width]}
        for name, spec in specs(width).items():
            if name in KINDS.get(kind, (kind, )):
                row[name] = measure(spec, device, prompts, batches, context, iters, log)
                torch.cuda.empty_cache()
        rows.append(row)
    print(json.dumps({"metric": "ragged-engine serving throughput, hybrid decoders beside the uniform one", "unit": "tokens/s",
                      "dtype": "bf16", "data": "synthetic tokens, random-init weights", "context": context,
                      "sizes": rows}), flush=True)
