#!/usr/bin/env python3
"""Flagship benchmark: Llama-2-7B ZeRO-3 bf16 training throughput (tokens/s) on N MI355X GPUs.

    python bench.py --gpus N --steps K --warmup W
For N>1 the driver launches one rank per GPU with torch.distributed.run (RCCL over xGMI); this script reads
RANK/LOCAL_RANK/WORLD_SIZE/MASTER_* from the environment.

Weak scaling: every rank runs the same micro-batch (global_batch = N x micro_batch x GAS sequences of seq_len
tokens). Synthetic uniform-random token ids, random-init weights of the real Llama-2-7B architecture (no network).
Each timed step is a full training step: forward, backward, gradient reduce-scatter, fused Adam on the fp32
partitions and parameter re-partitioning — nothing skipped. Prints ONE JSON line on rank 0.
"""
import argparse
import json
import os
import sys
import time

import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))


def parse():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=int(os.environ.get("WORLD_SIZE", "1")))
    ap.add_argument("--steps", type=int, default=5)
    ap.add_argument("--warmup", type=int, default=2)
    ap.add_argument("--model", default="llama2-7b", choices=["llama2-7b", "llama2-13b", "llama2-70b", "tiny"])
    ap.add_argument("--zero-init", action="store_true", help="construct the model inside zero.Init (ZeRO-3, >1 rank)")
    ap.add_argument("--offload-ratio", type=float, default=0.0,
                    help="ZeRO-Offload++ Twin-Flow: fraction of the fp32 master / Adam state kept in pinned host "
                         "memory and stepped by the native CPU Adam concurrently with the device Adam (BASELINE "
                         "config 4: Llama-2-70B ZeRO-3 + Twin-Flow)")
    ap.add_argument("--seq-len", type=int, default=4096)
    ap.add_argument("--micro-batch", type=int, default=int(os.environ.get("DS_BENCH_MB", "8")))
    ap.add_argument("--gas", type=int, default=1)
    ap.add_argument("--stage", type=int, default=3)
    ap.add_argument("--ckpt", action="store_true", help="activation checkpointing (not needed with 288 GB HBM)")
    ap.add_argument("--sp", type=int, default=1,
                    help="Ulysses sequence-parallel degree (BASELINE config: Llama-2 7B, seq 32k, sp over xGMI "
                         "all-to-all); dp = world / sp")
    ap.add_argument("--workload", default="train", choices=["train", "hybrid"],
                    help="train: the flagship training step (default); hybrid: serving throughput of hybrid decoders "
                         "beside the uniform one (benchmarks/hybrid_serving.py)")
    ap.add_argument("--sizes", default="2048,4096", help="--workload hybrid: model widths")
    ap.add_argument("--model-kind", default="both", choices=["hybrid", "perelorn", "uniform", "lefisun", "uniform_moe",
                                                           "nigilorn", "both", "moe", "close", "all"],
                    help="--workload hybrid")
    ap.add_argument("--local_rank", type=int, default=0)
    ap.add_argument("--host-dryrun", action="store_true",
                    help="CPU/gloo rehearsal of the multi-rank control flow (tiny model; not a measurement)")
    return ap.parse_args()


TUNED_GEMMS = os.path.join(os.path.dirname(os.path.abspath(__file__)), "profiles", "tunableop_llama7b_gfx950.csv")


def setup_gemm_tuning(on_gpu):
    """hipBLASLt/rocBLAS solution selection via PyTorch TunableOp. `DS_BENCH_TUNABLEOP=tune` measures every
    candidate solution for each GEMM shape of the step and records the winners in profiles/ (done once per
    model/config on an MI355X); the default `use` replays that table (no tuning inside the timed region)."""
    mode = os.environ.get("DS_BENCH_TUNABLEOP", "use")
    if not on_gpu or mode == "off":
        return
    tun = torch.cuda.tunable
    if mode == "tune":
        tun.enable(True)
        tun.tuning_enable(True)
        tun.set_max_tuning_duration(int(os.environ.get("DS_TUNABLEOP_MS", "30")))
        tun.set_max_tuning_iterations(int(os.environ.get("DS_TUNABLEOP_ITERS", "20")))
        out = os.environ.get("DS_TUNABLEOP_OUT", TUNED_GEMMS)
        if out != TUNED_GEMMS and os.path.exists(TUNED_GEMMS):
            import shutil
            os.makedirs(os.path.dirname(os.path.abspath(out)), exist_ok=True)
            shutil.copyfile(TUNED_GEMMS, out)  # keep the recorded shapes; only new ones get tuned
        tun.set_filename(out, False)
        if os.path.exists(out):
            tun.read_file(out)
        log(f"[bench] TunableOp tuning -> {out}")
        import threading

        def heartbeat():  # tuning a step's GEMM shapes takes minutes: keep the job visibly alive
            t0 = time.time()
            while True:
                time.sleep(30)
                log(f"[bench] tuning... {time.time() - t0:.0f}s, {len(tun.get_results())} shapes done")

        threading.Thread(target=heartbeat, daemon=True).start()
    elif os.path.exists(TUNED_GEMMS):
        tun.enable(True)
        tun.tuning_enable(False)
        tun.set_filename(TUNED_GEMMS, False)
        tun.read_file(TUNED_GEMMS)
        log(f"[bench] TunableOp replaying {TUNED_GEMMS}")


def log(*a):
    if int(os.environ.get("RANK", "0")) == 0:
        print(*a, file=sys.stderr, flush=True)


def causal_flops_per_token(cfg, seq_len):
    return 6 * cfg.num_params() + 6 * cfg.num_hidden_layers * cfg.hidden_size * seq_len


def forced_partition_loop(args, cfg, config, dev, batches, sync, steps=3, warmup=1):
    """tokens/s of the same model and config with DS_ZERO_FORCE_PARTITION=1 (a fresh engine; the first one's memory
    is released by the caller's references going away before this runs)."""
    import gc

    import deepspeedsyclsupport_amd as ds
    from deepspeedsyclsupport_amd.models.llama import LlamaForCausalLM
    main_engine = forced_partition_loop.release()
    del main_engine
    gc.collect()
    torch.cuda.empty_cache()
    os.environ["DS_ZERO_FORCE_PARTITION"] = "1"
    try:
        prev = torch.get_default_dtype()
        torch.set_default_dtype(torch.bfloat16)
        with torch.device(dev):
            model = LlamaForCausalLM(cfg)
        torch.set_default_dtype(prev)
        if args.ckpt:
            model.gradient_checkpointing_enable()
        engine, _, _, _ = ds.initialize(model=model, config=config)
        assert engine.optimizer.partition and engine.optimizer.coordinator is not None

        def step(i):
            x = batches[i % len(batches)]
            loss = engine(x, labels=x)
            engine.backward(loss)
            engine.step()
            return loss

        for i in range(warmup):
            step(i)
        sync()
        t0 = time.perf_counter()
        for i in range(steps):
            step(warmup + i)
        sync()
        dt = time.perf_counter() - t0
        return round(args.micro_batch * args.seq_len * steps / dt, 2)
    finally:
        os.environ["DS_ZERO_FORCE_PARTITION"] = "0"


def main():
    args = parse()
    if args.workload == "hybrid":
        from deepspeedsyclsupport_amd.benchmarks import hybrid_serving
        return hybrid_serving.run([int(w) for w in args.sizes.split(",")], args.model_kind, iters=2 * args.steps, log=log)
    import deepspeedsyclsupport_amd as ds
    from deepspeedsyclsupport_amd import comm as dist
    from deepspeedsyclsupport_amd.models.llama import (LlamaConfig, LlamaForCausalLM, llama2_7b_config, llama2_13b_config,
                                                       llama2_70b_config)

    ds.init_distributed(dist_backend="gloo" if args.host_dryrun else "nccl")
    rank, world = dist.get_rank(), dist.get_world_size()
    local = int(os.environ.get("LOCAL_RANK", "0"))
    if args.host_dryrun:
        dev = torch.device("cpu")
        args.model, args.seq_len, args.micro_batch = "tiny", min(args.seq_len, 128), min(args.micro_batch, 2)
    else:
        torch.cuda.set_device(local)
        dev = torch.device("cuda", local)
    on_gpu = dev.type == "cuda"
    setup_gemm_tuning(on_gpu)

    def sync():
        if on_gpu:
            torch.cuda.synchronize()

    def mem_gib(peak=False):
        if not on_gpu:
            return 0.0
        return (torch.cuda.max_memory_allocated() if peak else torch.cuda.memory_allocated()) / 2**30

    if args.model == "llama2-7b":
        cfg = llama2_7b_config(max_position_embeddings=args.seq_len)
    elif args.model == "llama2-13b":
        cfg = llama2_13b_config(max_position_embeddings=args.seq_len)
    elif args.model == "llama2-70b":
        cfg = llama2_70b_config(max_position_embeddings=args.seq_len)
    else:
        cfg = LlamaConfig(vocab_size=32000, hidden_size=1024, intermediate_size=2816, num_hidden_layers=4,
                          num_attention_heads=8, max_position_embeddings=args.seq_len)
    t0 = time.time()
    torch.manual_seed(1234)
    # build directly on the GPU in bf16 (fast init; fp32 masters are created by the ZeRO optimizer)
    prev = torch.get_default_dtype()
    torch.set_default_dtype(torch.bfloat16 if on_gpu else torch.float32)
    if (args.zero_init or args.model == "llama2-70b") and args.stage == 3 and world > 1:
        # built straight into ZeRO-3 partitions (zero.Init): 70B's 140 GB of bf16 weights never sit whole on a rank
        with ds.zero.Init(dtype=torch.bfloat16 if on_gpu else torch.float32), torch.device(dev):
            model = LlamaForCausalLM(cfg)
    else:
        with torch.device(dev):
            model = LlamaForCausalLM(cfg)
    torch.set_default_dtype(prev)
    if args.ckpt:
        model.gradient_checkpointing_enable()
    n_params = sum(p.numel() for p in model.parameters())
    log(f"[bench] built {args.model}: {n_params / 1e9:.3f}B params in {time.time() - t0:.1f}s")

    config = {
        "train_micro_batch_size_per_gpu": args.micro_batch,
        "gradient_accumulation_steps": args.gas,
        "steps_per_print": 10**9,
        "bf16": {"enabled": True},
        "gradient_clipping": 1.0,
        "optimizer": {"type": "AdamW", "params": {"lr": 1e-4, "betas": [0.9, 0.95], "eps": 1e-8,
                                                  "weight_decay": 0.1}},
        "zero_optimization": {
            "stage": args.stage,
            "overlap_comm": True,
            "contiguous_gradients": True,
            "reduce_bucket_size": int(2e8),
            "stage3_prefetch_bucket_size": int(2e8),
            "stage3_param_persistence_threshold": int(1e5),
            # sized for 288 GB of HBM: the whole bf16 model (13.4 GB at 7B) may stay gathered from a layer's forward
            # to its backward, so each partitioned parameter is all-gathered once per step, not twice
            "stage3_max_live_parameters": int(1e10),
            "stage3_max_reuse_distance": int(1e10),
        },
    }
    if args.offload_ratio > 0:
        config["zero_optimization"]["offload_optimizer"] = {"device": "cpu", "pin_memory": True,
                                                            "ratio": args.offload_ratio}
    assert world % args.sp == 0, "--sp must divide the number of ranks"
    dp = world // args.sp
    if args.sp > 1:
        config["sequence_parallel"] = {"size": args.sp}
        config["train_batch_size"] = dp * args.micro_batch * args.gas
    engine, _, _, _ = ds.initialize(model=model, config=config)
    sp_group = None
    if args.sp > 1:
        from deepspeedsyclsupport_amd.parallel import groups
        from deepspeedsyclsupport_amd.sequence.layer import enable_sequence_parallel, shard_sequence
        sp_group = groups._get_sequence_parallel_group()
        n_sp = enable_sequence_parallel(engine.module, sp_group)
        log(f"[bench] Ulysses sequence parallel sp={args.sp} dp={dp} on {n_sp} attention modules")
    log(f"[bench] engine ready in {time.time() - t0:.1f}s; mem {mem_gib():.1f} GiB")

    # every rank of one sequence-parallel group must see the same sequences (it keeps its own 1/sp slice)
    g = torch.Generator(device=dev).manual_seed(1000 + rank // args.sp)
    # a distinct synthetic batch for every micro-step (no repeated data for the model to memorise)
    n_micro = (args.warmup + args.steps) * args.gas
    batches = [torch.randint(0, cfg.vocab_size, (args.micro_batch, args.seq_len), device=dev, generator=g)
               for _ in range(n_micro)]

    def train_step(i):
        for a in range(args.gas):
            x = batches[i * args.gas + a]
            if sp_group is not None:
                inp, lab, off = shard_sequence(x, x, sp_group)
                loss = engine(inp, labels=lab, pos_offset=off, shift_labels=False)
            else:
                loss = engine(x, labels=x)
            engine.backward(loss)
            engine.step()
        return loss

    for i in range(args.warmup):
        tw = time.time()
        loss = train_step(i)
        sync()
        log(f"[bench] warmup {i}: loss={float(loss):.4f} {time.time() - tw:.2f}s peak {mem_gib(True):.1f} GiB")

    dist.barrier()
    sync()
    t_start = time.perf_counter()
    for i in range(args.steps):
        loss = train_step(args.warmup + i)
        if rank == 0 and (i + 1) % max(1, args.steps // 5) == 0:
            log(f"[bench] step {i + 1}/{args.steps}")
    sync()
    dist.barrier()
    elapsed = time.perf_counter() - t_start
    t = torch.tensor([elapsed], dtype=torch.float64, device=dev)
    dist.all_reduce(t, op=dist.ReduceOp.MAX)
    elapsed = float(t)

    # One data-parallel rank runs ZeRO-3 without partitioning (nothing to gather from): time a short second loop in
    # this process with the partitioned code path forced on (per-module all-gather on the prefetch stream,
    # reduce-scatter on the reduction stream, shard pointing), so the multi-rank machinery is measured at N=1 too.
    forced = None
    final_loss = float(loss)
    holder = {"engine": engine, "model": model}

    def release():
        return holder.pop("engine", None), holder.pop("model", None)

    forced_partition_loop.release = release
    partitioned = bool(getattr(engine.optimizer, "partition", False))
    if world == 1 and on_gpu and args.stage == 3 and not args.host_dryrun and \
            os.environ.get("DS_ZERO_FORCE_PARTITION", "0") != "1" and os.environ.get("DS_BENCH_FORCED", "1") == "1":
        try:
            if args.gas == 1 and args.sp == 1 and args.offload_ratio == 0:
                del engine, model, loss
                forced = forced_partition_loop(args, cfg, config, dev, batches, sync)
        except Exception as e:  # the headline number above stands on its own
            log(f"[bench] forced-partition loop failed: {type(e).__name__}: {e}")

    ms_per_step = elapsed / args.steps * 1e3
    tokens_per_step = dp * args.micro_batch * args.gas * args.seq_len  # each sp group covers whole sequences
    tok_s = tokens_per_step * args.steps / elapsed
    flops_tok = cfg.flops_per_token(args.seq_len)
    tflops_gpu = tok_s * flops_tok / world / 1e12
    peak_mem = mem_gib(True)
    if rank == 0:
        out = {
            "metric": "tokens/sec Llama-2-7B ZeRO-3 at 1/2/4/8 MI355X; peak trainable params/GPU",
            "value": round(tok_s, 2),
            "unit": "tokens/s",
            "n_gpus": world,
            "steps": args.steps,
            "warmup": args.warmup,
            "ms_per_step": round(ms_per_step, 2),
            "higher_is_better": True,
            "scaling": "weak",
            "vs_baseline": None,
            "dtype": "bf16",
            "data": "synthetic (uniform random token ids, random-init weights)",
            "config": {
                "model": {"llama2-7b": "Llama-2-7B", "llama2-13b": "Llama-2-13B", "llama2-70b": "Llama-2-70B",
                          "tiny": "llama-tiny"}[args.model],
                "global_batch": dp * args.micro_batch * args.gas,
                "seq_len": args.seq_len,
                "parallelism": f"dp{dp}" + (f"-sp{args.sp}" if args.sp > 1 else ""),
                "zero_stage": args.stage,
                # True when parameters / gradients really are partitioned and gathered / reduce-scattered in the
                # timed steps (always with > 1 data-parallel rank; at one rank only with DS_ZERO_FORCE_PARTITION=1)
                "zero_partitioned": partitioned,
                "twin_flow_offload_ratio": args.offload_ratio,
                "attention": "in-tree CDNA4 flash fwd+bwd (csrc/attn/flash_{fwd,bwd}.hip)",
                "micro_batch_per_gpu": args.micro_batch,
                "gradient_accumulation_steps": args.gas,
                "activation_checkpointing": bool(args.ckpt),
                "optimizer": "FusedAdam(AdamW, gfx950 kernel)",
            },
            "tokens_per_sec_per_gpu": round(tok_s / world, 2),
            # model FLOPs with the usual full-attention convention (12*L*H*S per token), and with the causal mask
            # accounted for (half of the score / context FLOPs are never computed)
            "model_tflops_per_gpu": round(tflops_gpu, 1),
            "mfu_vs_2.5PF_bf16_dense": round(tflops_gpu / 2500.0, 4),
            "model_tflops_per_gpu_causal": round(tok_s * causal_flops_per_token(cfg, args.seq_len) / world / 1e12, 1),
            "mfu_causal_vs_2.5PF_bf16_dense": round(tok_s * causal_flops_per_token(cfg, args.seq_len) / world / 2.5e15,
                                                    4),
            "forced_partition_tokens_per_sec": forced,
            "params": n_params,
            "peak_mem_gib_per_gpu": round(peak_mem, 1),
            "final_loss": round(final_loss, 4),
        }
        print(json.dumps(out), flush=True)
    dist.barrier()


if __name__ == "__main__":
    main()
