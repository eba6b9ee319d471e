"""Replay of a recorded request trace through the ragged engine, step by step, writing the logits it asks for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N  < steps

Each line of standard input is one step, a JSON object {"step": i, "entries": [{"id": .., "tokens": [..], "want":
[..]}], "end": [..]}: the entries' next tokens run as ONE ragged batch (`InferenceEngineV2.put`), the logits at the
places named by `want` go to DIR/<step>.f32 (little-endian fp32, [wanted, vocab]), the requests in `end` are flushed,
and "done <step>" is printed. Nothing is sampled."""
import argparse
import json
import os
import sys

import torch

from .config_v2 import AllocationMode, RaggedInferenceEngineConfig
from .engine_factory import build_hf_engine

BLOCK = 64
MAX_LIVE = 4


def trace_engine(model, dtype, max_tokens, max_live=MAX_LIVE):
    """An engine whose pools hold `max_tokens` cached tokens and `max_live` sequences, no more."""
    blocks = max(-(-max_tokens // BLOCK), 1)
    cfg = RaggedInferenceEngineConfig(
        state_manager={"memory_config": {"mode": AllocationMode.ALLOCATE, "size": blocks},
                       "max_tracked_sequences": max_live, "max_ragged_sequence_count": max_live,
                       "max_ragged_batch_size": max(blocks * BLOCK, max_live), "max_context": blocks * BLOCK,
                       "state_slots": max_live},
        kv_cache={"block_size": BLOCK})
    return build_hf_engine(model, cfg, dtype=dtype)


class TraceRunner:

    def __init__(self, engine, out_dir):
        self.engine, self.out_dir = engine, out_dir
        self.uids, self._next = {}, 0

    def _uid(self, rid):
        if rid not in self.uids:
            self.uids[rid] = self._next
            self._next += 1
        return self.uids[rid]

    def step(self, rec):
        """Run one step; returns the wanted logits [n, vocab] fp32 on the host (None if nothing was wanted)."""
        entries = [e for e in rec["entries"] if e["tokens"]]
        logits = None
        if entries:
            want = [e.get("want", []) for e in entries]
            logits = self.engine.put([self._uid(e["id"]) for e in entries],
                                     [torch.tensor(e["tokens"], dtype=torch.long) for e in entries],
                                     logit_positions=want)
            logits = logits.float().cpu() if any(want) else None
        for rid in rec.get("end", []):
            if rid in self.uids:
                self.engine.flush(self.uids.pop(rid))
        return logits

    def run(self, lines, write):
        for line in lines:
            if not line.strip():
                continue
            rec = json.loads(line)
            logits = self.step(rec)
            if logits is not None:
                logits.numpy().astype("<f4").tofile(os.path.join(self.out_dir, f"{rec['step']}.f32"))
            write(f"done {rec['step']}")


def main(argv=None):
    ap = argparse.ArgumentParser(description="Replay a request trace through the ragged engine")
    ap.add_argument("--model", required=True, help="checkpoint directory (config.json, model.safetensors)")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="directory for the <step>.f32 files")
    ap.add_argument("--max-tokens", type=int, required=True, help="cached tokens the engine must hold at once")
    args = ap.parse_args(argv)
    if not torch.cuda.is_available():
        sys.exit("trace_run needs a HIP device")
    torch.backends.cuda.matmul.allow_tf32 = False
    torch.set_float32_matmul_precision("highest")
    os.makedirs(args.out, exist_ok=True)
    engine = trace_engine(args.model, getattr(torch, args.dtype), args.max_tokens)

    def write(line):
        sys.stdout.write(line + "\n")
        sys.stdout.flush()

    TraceRunner(engine, args.out).run(sys.stdin, write)
    torch.cuda.synchronize()


if __name__ == "__main__":
    main()
