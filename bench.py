#!/usr/bin/env python3
"""Flagship benchmark: end-to-end n-way consensus serving on MI355X.

Measures the BASELINE.json headline metric — end-to-end consensus requests/sec
(and per-request latency) at n=5 on Llama-3-8B TP=1 — on synthetic prompts and
random-init weights (no network). Each timed step serves a fixed batch of
consensus requests END TO END **through the public client API**
(``AsyncKLLMs().chat.completions.create`` — the literal L4 contract,
reference k_llms/client.py:31-72): concurrent create() calls merge in the
continuous-batching scheduler (shared prefill, n fanned decode streams per
request, HIP kernels, paged KV, hipGraph decode), and each call returns a
consolidated KLLMsChatCompletion with likelihoods — consensus inside the
timed region.

Configs:
  --config llama8b   (default) chat.completions.create n=5, Llama-3-8B
  --config parse16   chat.completions.parse, nested Pydantic schema,
                     n=16 + likelihoods
  --config mixtral8  Mixtral-8x7B parse() n=8
  --config llama70b  Llama-3-70B create n=5 (TP=8 with
                     --parallel tp under an 8-rank launch)

Multi-GPU (--gpus N, launched by torch.distributed.run with one rank per GPU):
default is data-parallel weak scaling — each rank runs an independent TP=1
engine serving its own request stream; the reported value is the whole-job
aggregate. ``--parallel tp`` instead shards ONE engine across all ranks
(column/row-parallel layers + RCCL/xGMI all-reduce): rank 0 runs the client
and scheduler, other ranks follow in lockstep (parallel/serve.py).

``--compare-families`` is a separate, single-GPU measurement: prefill and
decode token throughput of the listed-layer families (Zutalix, Medilix,
Mitunex, Pironex, Bavesun; ``--families`` picks) beside
the dense Llama stack of the same width / depth / heads / ff, straight through
LLMEngine.generate (random-init weights, synthetic token ids). It prints its
own JSON line and leaves the default workload untouched.

Usage: python bench.py [--gpus N] [--steps K] [--warmup W]
Rank 0 prints exactly one JSON result line.
"""

import argparse
import asyncio
import json
import os
import sys
import time

import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

REFERENCE_BASELINE = {
    # BASELINE.md rows (remote OpenAI API numbers, context bar)
    "llama8b": 1.2,    # consensus n=3 throughput (req/s)
    "llama70b": 1.2,
    "parse16": 0.7,    # structured output throughput
    "mixtral8": 0.7,
}


def log(msg):
    if int(os.environ.get("RANK", "0")) == 0:
        print(msg, file=sys.stderr, flush=True)


def _mean_likelihood(node) -> float:
    """Average of all leaf confidences — the reference's 'consensus quality'
    scale (README_TESTS.md:269-273: 0.8-0.9 good)."""
    leaves = []

    def walk(v):
        if isinstance(v, dict):
            for x in v.values():
                walk(x)
        elif isinstance(v, (list, tuple)):
            for x in v:
                walk(x)
        elif isinstance(v, (int, float)):
            leaves.append(float(v))

    walk(node)
    return sum(leaves) / len(leaves) if leaves else 0.0


def _enable_tunableop(local_rank: int) -> None:
    """Load the shipped offline GEMM tuning results (read-only). The decode-
    shape GEMMs (M = graph bucket) are ~30% faster under the tuned algorithm
    picks than the default heuristics (see kllms_amd/tunableop/)."""
    import shutil
    import tempfile

    shipped = os.path.join(os.path.dirname(os.path.abspath(__file__)),
                           "kllms_amd", "tunableop", "tunableop_gfx9500.csv")
    if not os.path.exists(shipped):
        return
    tmp = tempfile.mkdtemp(prefix="kllms_tunableop_")
    # TunableOp inserts the device ordinal before ".csv"; provide every ordinal
    for i in range(8):
        shutil.copy(shipped, os.path.join(tmp, f"tunableop_gfx950{i}.csv"))
    try:
        torch.cuda.tunable.enable(True)
        # KLLMS_TUNE=1 re-runs the offline tuning and leaves results in the
        # temp dir (printed) for refreshing kllms_amd/tunableop/.
        tune = os.environ.get("KLLMS_TUNE", "0") == "1"
        torch.cuda.tunable.tuning_enable(tune)
        torch.cuda.tunable.set_filename(os.path.join(tmp, "tunableop_gfx950.csv"), insert_device_ordinal=True)
        torch.cuda.tunable.read_file()
        if tune:
            log(f"[bench] tunableop TUNING, results dir: {tmp}")
            import atexit

            atexit.register(torch.cuda.tunable.write_file)
            atexit.register(lambda: log(f"[bench] tuned results in {tmp}"))
    except Exception as e:
        log(f"[bench] tunableop disabled ({e})")


def make_prompt(rank: int, step: int, i: int, prompt_len_tokens: int) -> str:
    # deterministic synthetic prompt of roughly prompt_len_tokens byte-tokens
    seedtxt = f"Request {rank}-{step}-{i}: extract the entities. "
    body = ("The quick brown fox jumps over the lazy dog near the riverbank. " * 200)
    return (seedtxt + body)[:prompt_len_tokens]


def make_schema():
    """Nested Pydantic schema for parse() configs (mirrors the reference's
    Company/Department test shape, README_TESTS.md:63-73). Fields carry
    bounds (maxLength / maxItems / integer ranges) so the byte DFA forces
    structurally complete objects in a bounded token budget — on random-init
    weights an unbounded field would run to the max_tokens cap instead of
    closing (an earlier schema_valid caveat)."""
    from typing import List

    from pydantic import BaseModel, Field

    class Employee(BaseModel):
        name: str = Field(max_length=16)
        role: str = Field(max_length=12)

    class Department(BaseModel):
        name: str = Field(max_length=16)
        headcount: int = Field(ge=0, le=9999)
        employees: List[Employee] = Field(max_length=2)

    class Company(BaseModel):
        company: str = Field(max_length=20)
        founded: int = Field(ge=0, le=9999)  # range the digit-count DFA bound can honor
        departments: List[Department] = Field(max_length=2)

    return Company


CONFIG_DEFAULTS = {
    # model, n, mode, batch, max_new
    "llama8b": dict(model="llama-3-8b", n=5, mode="create", batch=24, max_new=64),
    "parse16": dict(model="llama-3-8b", n=16, mode="parse", batch=4, max_new=352),
    "mixtral8": dict(model="mixtral-8x7b", n=8, mode="parse", batch=8, max_new=352),
    "llama70b": dict(model="llama-3-70b", n=5, mode="create", batch=4, max_new=64),
}


def compare_families(args) -> None:
    """Prefill / decode tokens per second of the two families at equal layer
    shapes. One engine at a time; W warmup + K timed generate() calls each."""
    from kllms_amd.engine.config import MODEL_PRESETS, EngineConfig
    from kllms_amd.engine.engine import GenRequest, LLMEngine
    from kllms_amd.engine.sampling import SamplingParams

    device = "cuda:0" if torch.cuda.is_available() else "cpu"
    sizes = [s for s in args.sizes.split(",") if s]
    B, P, N = args.batch or 16, args.prompt_len, args.max_new or 64
    rows = []
    for size in sizes:
        for fam in [f for f in args.families.split(",") if f]:
            name = f"{fam}-{size}" if f"{fam}-{size}" in MODEL_PRESETS else f"{size}-{fam}"
            kw = dict(model=name, device=device, seed=0, use_hip_graphs=device != "cpu" and not args.no_graphs,
                      max_seq_len=P + N + 64, max_batch_size=max(B, 8), enable_prefix_caching=False,
                      eos_token_id=-1)     # no stop id: every stream decodes its N tokens
            if device == "cpu":
                kw["max_kv_blocks"] = 4096
            eng = LLMEngine(EngineConfig(**kw))
            g = torch.Generator().manual_seed(1)
            mk = lambda: [GenRequest(prompt_ids=torch.randint(3, 250, (P,), generator=g).tolist(), n=1,
                                     sampling=SamplingParams(temperature=1.0, max_tokens=N, seed=i))
                          for i in range(B)]
            pre = dec = 0.0
            steps = 0
            for it in range(args.warmup + args.steps):
                eng.generate(mk())
                if it >= args.warmup:
                    t = eng.last_timings
                    pre += t["prefill_ms"]
                    dec += t["decode_ms"]
                    steps += t["decode_steps"]
            row = {"model": name, "batch": B, "prompt_len": P,
                   "prefill_tok_s": round(B * P * args.steps / (pre / 1e3), 1),
                   "decode_tok_s": round(B * steps / (dec / 1e3), 1),
                   "prefill_ms": round(pre / args.steps, 2),
                   "decode_ms_per_step": round(dec / max(1, steps), 3)}
            log(f"[compare] {row}")
            rows.append(row)
            del eng
            if device != "cpu":
                torch.cuda.empty_cache()
    print(json.dumps({"metric": "family_compare_tokens_per_s", "unit": "tok/s", "dtype": "bf16" if device != "cpu" else "fp32",
                      "data": "synthetic", "steps": args.steps, "warmup": args.warmup, "rows": rows}), flush=True)


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--compare-families", action="store_true",
                    help="prefill/decode tok/s of the hybrid families beside the dense Llama stack of equal shape")
    ap.add_argument("--families", type=str, default="llama,zutalix,medilix",
                    help="--compare-families: model families to time, in order "
                         "(llama, zutalix, medilix, mitunex, pironex, bavesun, dimuvik)")
    ap.add_argument("--sizes", type=str, default="1b-l6,8b-l6", help="--compare-families: preset size suffixes")
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=3)
    ap.add_argument("--warmup", type=int, default=1)
    ap.add_argument("--config", type=str, default="llama8b", choices=list(CONFIG_DEFAULTS))
    ap.add_argument("--model", type=str, default=None)
    ap.add_argument("--n", type=int, default=None)
    ap.add_argument("--batch", type=int, default=None, help="consensus requests per step per engine")
    ap.add_argument("--prompt-len", type=int, default=512, help="approx prompt tokens")
    ap.add_argument("--max-new", type=int, default=None, help="decode tokens per stream")
    ap.add_argument("--no-graphs", action="store_true")
    ap.add_argument("--parallel", type=str, default="dp", choices=["dp", "tp"],
                    help="dp: one engine per rank (weak scaling); tp: ONE engine sharded over all ranks")
    args = ap.parse_args()
    if args.compare_families:
        compare_families(args)
        return

    cfgd = CONFIG_DEFAULTS[args.config]
    model = args.model or cfgd["model"]
    n = args.n if args.n is not None else cfgd["n"]
    batch = args.batch if args.batch is not None else cfgd["batch"]
    max_new = args.max_new if args.max_new is not None else cfgd["max_new"]
    mode = cfgd["mode"]

    world_size = int(os.environ.get("WORLD_SIZE", "1"))
    rank = int(os.environ.get("RANK", "0"))
    local_rank = int(os.environ.get("LOCAL_RANK", "0"))
    on_gpu = torch.cuda.is_available()
    dist = None
    if world_size > 1:
        import torch.distributed as dist_mod

        dist = dist_mod
        backend = "nccl" if on_gpu else "gloo"
        dist.init_process_group(backend=backend)
        if on_gpu:
            torch.cuda.set_device(local_rank)

    device = f"cuda:{local_rank}" if on_gpu else "cpu"
    tp_mode = args.parallel == "tp" and world_size > 1

    if on_gpu:
        _enable_tunableop(local_rank)

    from kllms_amd import AsyncKLLMs

    log(f"[bench] building engine: {model} on {device} ({'tp' + str(world_size) if tp_mode else 'tp1'})")
    t_build = time.perf_counter()
    client_kwargs = dict(
        model=model,
        device=device,
        use_hip_graphs=(on_gpu and not args.no_graphs),
        seed=0 if tp_mode else rank,
        default_max_new_tokens=max_new,
        max_seq_len=max(1024, args.prompt_len + max_new + 64),
    )
    if tp_mode:
        client_kwargs["tp_size"] = world_size
    if not on_gpu:
        client_kwargs["max_kv_blocks"] = 4096

    follower = None
    if tp_mode and rank != 0:
        # non-zero TP ranks run the lockstep follower loop; rank 0 drives the
        # public client below and broadcasts every engine action.
        from kllms_amd.engine.api import LocalEngineClient
        from kllms_amd.parallel.serve import TPFollower

        eng_client = LocalEngineClient(**client_kwargs)
        follower = TPFollower(eng_client.engine)
        log(f"[bench] rank {rank}: follower ready in {time.perf_counter() - t_build:.1f}s")
        follower.run()  # blocks until rank 0 sends stop
        if dist is not None:
            dist.barrier()
            dist.destroy_process_group()
        return

    k = AsyncKLLMs(**client_kwargs)
    eng_client = k.client
    _ = eng_client.engine  # materialize weights now
    if tp_mode:
        from kllms_amd.parallel.serve import TPCoordinator

        eng_client.scheduler.coordinator = TPCoordinator(eng_client.engine)
    log(f"[bench] engine ready in {time.perf_counter() - t_build:.1f}s")

    schema = make_schema() if mode == "parse" else None
    quality_scores: list = []
    schema_valid = [0, 0]

    async def one_request(step_idx: int, i: int):
        msgs = [{"role": "user", "content": make_prompt(rank, step_idx, i, args.prompt_len)}]
        seed = 10_000 * rank + 100 * step_idx + i
        if mode == "parse":
            res = await k.chat.completions.parse(
                messages=msgs, model=model, response_format=schema,
                n=n, temperature=0.9, max_tokens=max_new, seed=seed,
            )
            for ch in res.choices[1:]:
                schema_valid[1] += 1
                if ch.message.parsed is not None:
                    schema_valid[0] += 1
        else:
            res = await k.chat.completions.create(
                messages=msgs, model=model,
                n=n, temperature=0.8, max_tokens=max_new, seed=seed,
            )
        quality_scores.append(_mean_likelihood(res.likelihoods))
        return res

    prev_stats = {}

    async def run_step(step_idx: int):
        import time as _t
        t0 = _t.perf_counter()
        await asyncio.gather(*(one_request(step_idx, i) for i in range(batch)))
        if os.environ.get("KLLMS_BENCH_VERBOSE"):
            sched = getattr(eng_client, "_scheduler", None)
            cur = dict(sched.stats) if sched else {}
            delta = {k: round(v - prev_stats.get(k, 0), 4) if isinstance(v, float)
                     else v - prev_stats.get(k, 0) for k, v in cur.items()}
            prev_stats.clear()
            prev_stats.update(cur)
            pc = getattr(eng_client.engine, "prefix_cache", None)
            log(f"[bench] step {step_idx}: wall={_t.perf_counter()-t0:.3f}s "
                f"sched_delta={delta} prefix={pc.stats if pc else None}")

    def barrier_sync():
        if dist is not None and not tp_mode:
            dist.barrier()
        if on_gpu:
            torch.cuda.synchronize()

    async def timed_run():
        # ONE event loop (and one to_thread pool) for the whole bench;
        # asyncio's default executor caps at 32 threads, which would split
        # a >32-request burst into two admission waves — size it to the batch
        import concurrent.futures as _cf
        asyncio.get_running_loop().set_default_executor(
            _cf.ThreadPoolExecutor(max_workers=batch + 8))
        for w in range(args.warmup):
            log(f"[bench] warmup {w + 1}/{args.warmup}")
            await run_step(-1 - w)
        barrier_sync()
        t0 = time.perf_counter()
        for s in range(args.steps):
            await run_step(s)
        barrier_sync()
        return time.perf_counter() - t0

    elapsed = asyncio.run(timed_run())

    # MAX over ranks (DP mode; in TP mode only rank 0 times the job)
    if dist is not None and not tp_mode:
        t = torch.tensor([elapsed], dtype=torch.float64,
                         device=device if dist.get_backend() == "nccl" else "cpu")
        dist.all_reduce(t, op=dist.ReduceOp.MAX)
        elapsed = float(t.item())

    n_engines = 1 if tp_mode else world_size
    total_requests = args.steps * batch * n_engines
    value = total_requests / elapsed
    ms_per_step = elapsed / args.steps * 1000.0

    if rank == 0:
        config = {
            "model": model,
            "n": n,
            "mode": mode,
            "global_batch": batch * n_engines,
            "seq_len": args.prompt_len,
            "max_new_tokens": max_new,
            "parallelism": f"tp{world_size}" if tp_mode else f"dp{world_size} tp1",
            "api_path": "AsyncKLLMs.chat.completions." + ("parse" if mode == "parse" else "create"),
            "completions_per_s": round(value * n, 3),
            # amortized (throughput) latency and the user-perceived batch
            # wall time (a sync batch's requests all complete together)
            "consensus_latency_s_per_request": round(elapsed / (args.steps * batch), 4),
            "batch_wall_s": round(ms_per_step / 1000.0, 4),
            "mean_consensus_quality": round(sum(quality_scores) / len(quality_scores), 4) if quality_scores else None,
        }
        if mode == "parse":
            config["schema_valid_fraction"] = round(schema_valid[0] / max(1, schema_valid[1]), 4)
        result = {
            "metric": "end_to_end_consensus_requests_per_s",
            "value": round(value, 4),
            "unit": "req/s",
            "n_gpus": world_size,
            "steps": args.steps,
            "warmup": args.warmup,
            "ms_per_step": round(ms_per_step, 2),
            "higher_is_better": True,
            "scaling": "weak" if not tp_mode else "strong",
            "vs_baseline": round(value / REFERENCE_BASELINE[args.config], 3),
            "dtype": "bf16" if on_gpu else "float32",
            "data": "synthetic prompts, random-init weights",
            "config": config,
        }
        print(json.dumps(result), flush=True)

    if tp_mode:
        sched = eng_client.scheduler
        coord = sched.coordinator
        sched.shutdown()      # join the worker thread first …
        coord.stop()          # … then release the followers
    elif getattr(eng_client, "_scheduler", None) is not None:
        eng_client._scheduler.shutdown()   # no worker thread is left running torch code at interpreter exit
    if dist is not None:
        dist.barrier()
        dist.destroy_process_group()


if __name__ == "__main__":
    main()
