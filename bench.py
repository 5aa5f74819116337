#!/usr/bin/env python3
"""Flagship serving benchmark (driver contract).

Measures the BASELINE.json metric — routed req/s + p50 EPP latency + P/D
goodput (tok/s under TTFT SLO) on Llama-3-8B bf16 — on N GPUs of one node:
one rank per GPU (torchrun), rank 0 runs the router (EPP) on top of its
worker, every rank runs a continuous-batching engine; synthetic
shared-prefix prompts with random-init weights (no network for datasets or
checkpoints).

  python bench.py --gpus N --steps K --warmup W [--mode mono|pd|fc]

A "step" is one node iteration (engine decode iteration + any scheduled
prefill chunk + one control-plane exchange). The timed region brackets
EXACTLY K steps with a barrier + torch.cuda.synchronize on both sides; the
reported value is the WHOLE-JOB aggregate SLO-goodput tok/s over all ranks
(MAX of per-rank elapsed used as the denominator).
"""
import argparse
import json
import os
import random
import sys
import time

import numpy as np
import torch


def parse_args():
    p = argparse.ArgumentParser()
    p.add_argument("--gpus", type=int, default=1)
    p.add_argument("--steps", type=int, default=200)
    p.add_argument("--warmup", type=int, default=40)
    p.add_argument("--mode", default="mono",
                   choices=["mono", "pd", "fc", "epd", "layers"],
                   help="mono=prefix-aware DP decode; pd=P/D disagg; "
                        "fc=flow control at overload; epd=E/P/D multimodal; "
                        "layers=prefill and decode of a layer-listed "
                        "design beside Llama layers of equal size (one GPU)")
    p.add_argument("--layer-design", default="rururax",
                   choices=["rururax", "sezazen"],
                   help="design of --mode layers")
    p.add_argument("--layer-sizes", default="2b,8b,32b",
                   help="sizes of --mode layers, comma-separated")
    p.add_argument("--model", default="llama-3-8b",
                   help="llama-3-8b | qwen3-32b (the reference regression model) "
                        "| any registered name or checkpoint folder")
    # the reference's regression harness shape: input 1024 / output 1024
    # (config/manifests/regression-testing/single-workload-regression.yaml)
    p.add_argument("--prompt-len", type=int, default=1024)
    p.add_argument("--max-tokens", type=int, default=1024)
    p.add_argument("--concurrency", type=int, default=256,
                   help="in-flight requests per decode rank (closed loop; "
                        "256 is the measured single-GPU knee at the "
                        "in=1024/out=1024 reference shape)")
    p.add_argument("--shared-prefix", type=float, default=0.5,
                   help="fraction of prompt shared within a request group")
    p.add_argument("--group", type=int, default=4,
                   help="requests per shared-prefix group")
    p.add_argument("--kv-gb", type=float, default=160.0,
                   help="KV pool budget per GPU (GB; MI355X has 288)")
    p.add_argument("--kv-dtype", default="auto",
                   choices=["auto", "bf16", "fp8"],
                   help="KV cache storage dtype (fp8 = OCP e4m3; compute "
                        "stays bf16)")
    p.add_argument("--arrival-rate", type=float, default=0.0,
                   help="open-loop Poisson arrivals (req/s, whole node); "
                        "0 = closed loop at --concurrency. The reference's "
                        "regression harness sweeps this rate "
                        "(single-workload-regression.yaml:30-45)")
    p.add_argument("--ttft-slo-ms", type=float, default=2000.0)
    p.add_argument("--device", default=None, help="override (cpu for tests)")
    p.add_argument("--seed", type=int, default=1234)
    return p.parse_args()


def pd_topology(n: int) -> str:
    if n < 2:
        return "mono"
    prefill = max(1, n // 4)
    return f"pd:{prefill}p{n - prefill}d"


def epd_topology(n: int) -> str:
    # 1 encode + 2 prefill + 5 decode at n=8
    if n < 3:
        return pd_topology(n)
    prefill = max(1, (n - 1) // 3)
    return f"epd:1e{prefill}p{n - 1 - prefill}d"


EPD_YAML = """
plugins:
  - type: decode-filter
  - type: prefill-filter
  - type: encode-filter
  - type: queue-scorer
  - type: kv-cache-utilization-scorer
  - type: prefix-cache-scorer
  - type: max-score-picker
  - type: prefix-based-pd-decider
    parameters: {nonCachedTokens: 256}
  - type: always-disagg-multimodal-decider
  - type: disagg-profile-handler
    parameters:
      pdDecider: prefix-based-pd-decider
      encodeDecider: always-disagg-multimodal-decider
schedulingProfiles:
  - name: decode
    plugins:
      - {pluginRef: decode-filter}
      - {pluginRef: prefix-cache-scorer, weight: 3}
      - {pluginRef: queue-scorer, weight: 1}
      - {pluginRef: kv-cache-utilization-scorer, weight: 1}
      - {pluginRef: max-score-picker}
  - name: prefill
    plugins:
      - {pluginRef: prefill-filter}
      - {pluginRef: queue-scorer, weight: 1}
      - {pluginRef: max-score-picker}
  - name: encode
    plugins:
      - {pluginRef: encode-filter}
      - {pluginRef: queue-scorer, weight: 1}
      - {pluginRef: max-score-picker}
"""


class Workload:
    """Deterministic shared-prefix synthetic prompt stream."""

    def __init__(self, args, vocab=128000):
        self.args = args
        self.rng = random.Random(args.seed)
        self.vocab = vocab
        self.n_issued = 0
        self._group_prefix = None

    def next_request(self):
        from llm_d_inference_scheduler_amd.scheduling.types import LLMRequest
        a = self.args
        i = self.n_issued
        self.n_issued += 1
        shared = int(a.prompt_len * a.shared_prefix)
        if i % a.group == 0 or self._group_prefix is None:
            self._group_prefix = [self.rng.randrange(256, self.vocab)
                                  for _ in range(shared)]
        tokens = self._group_prefix + \
            [self.rng.randrange(256, self.vocab)
             for _ in range(a.prompt_len - shared)]
        req = LLMRequest(request_id=f"req-{i}", model=a.model,
                         prompt_tokens=tokens, max_tokens=a.max_tokens,
                         prompt="")
        req.ttft_slo_ms = a.ttft_slo_ms
        if a.mode == "epd":
            from llm_d_inference_scheduler_amd.scheduling.types import \
                MultiModalItem
            # 1 image per request from a small URL pool (dedupe-friendly)
            req.mm_items = [MultiModalItem("image_url",
                                           f"http://img/{i % 16}")]
        if a.mode == "fc":
            # mixed-SLO priority tiers: 1/3 critical, 1/3 standard,
            # 1/3 sheddable batch (InferenceObjective priorities)
            tier = i % 3
            req.objective_name = ["critical", "standard", "batch"][tier]
            req.fairness_id = f"tenant-{i % 4}"
        return req


def main():
    args = parse_args()
    if args.mode == "layers":
        return layers_main(args)
    wd = float(os.environ.get("LLMD_BENCH_WATCHDOG", "0"))
    if wd > 0:
        # debug: dump all thread stacks and die if the run wedges
        import faulthandler
        faulthandler.dump_traceback_later(wd, exit=True)
    rank = int(os.environ.get("RANK", "0"))
    world = int(os.environ.get("WORLD_SIZE", "1"))
    local_rank = int(os.environ.get("LOCAL_RANK", str(rank)))
    if world == 1 and args.gpus > 1:
        print("ERROR: multi-GPU bench must be launched via torchrun",
              file=sys.stderr)
        sys.exit(2)

    use_gpu = torch.cuda.is_available() if args.device is None \
        else args.device.startswith("cuda")
    # oversubscribed rig: more ranks than visible GPUs (e.g. a 2-rank P/D
    # topology exercised on a 1-GPU box) — all ranks share cuda:0, the
    # process group is gloo (RCCL cannot host two ranks on one device) and
    # KV moves via the HIP-IPC peer-pull transport, which needs no RCCL
    n_vis = torch.cuda.device_count() if use_gpu else 0
    same_dev = use_gpu and world > n_vis
    device = (args.device or
              ("cuda:0" if same_dev else
               (f"cuda:{local_rank}" if use_gpu else "cpu")))
    dtype = torch.bfloat16 if use_gpu else torch.float32

    import torch.distributed as dist
    mailbox_group = transfer_group = None
    if world > 1:
        backend = "nccl" if use_gpu and not same_dev else "gloo"
        if use_gpu and not same_dev:
            torch.cuda.set_device(local_rank)
        dist.init_process_group(backend)
        transfer_group = None  # default group (RCCL over xGMI)
        mailbox_group = dist.new_group(backend="gloo")
        # bench-level control collectives get their OWN gloo group: the
        # mailbox group now runs a pipelined exchange on a helper thread,
        # and concurrent collectives on one gloo group are unordered
        ctrl_group = dist.new_group(backend="gloo")
    else:
        ctrl_group = None

    from llm_d_inference_scheduler_amd.models import registry
    from llm_d_inference_scheduler_amd.models.configs import (
        LLAVA_1_5_7B_TEXT, TINY_LLAMA, TINY_LLAVA)
    from llm_d_inference_scheduler_amd.node import NodeConfig, NodeRunner
    from llm_d_inference_scheduler_amd.flowcontrol import BandConfig
    from llm_d_inference_scheduler_amd.api.objectives import InferenceObjective

    if same_dev:
        # all ranks share one 288 GB GPU: shrink each rank's KV budget so
        # world * (weights + KV + activations) fits
        args.kv_gb = min(args.kv_gb, max(16.0, 288.0 / world - 48.0))

    model_cfg = registry.resolve(args.model) if os.path.isdir(args.model) \
        else registry.MODELS.get(args.model, TINY_LLAMA)
    if args.mode == "epd":
        model_cfg = LLAVA_1_5_7B_TEXT  # BASELINE config 5 multimodal model
        args.model = model_cfg.name
    if not use_gpu and args.model in ("llama-3-8b", "qwen3-32b",
                                      "llava-1.5-7b"):
        # CPU smoke of the bench harness itself uses the tiny config; a GPU
        # run always uses the full flagship model (anything else is invalid
        # for reporting).
        from llm_d_inference_scheduler_amd.models.configs import TINY_QWEN
        model_cfg = (TINY_LLAVA if args.mode == "epd" else
                     TINY_QWEN if args.model == "qwen3-32b" else TINY_LLAMA)
        args.prompt_len = min(args.prompt_len, 96)
        args.max_tokens = min(args.max_tokens, 8)
        args.concurrency = min(args.concurrency, 8)

    topology = "mono"
    parallelism = f"dp{world}"
    epp_yaml = ""
    if args.mode == "pd" and world >= 2:
        topology = pd_topology(world)
        parallelism = topology
    elif args.mode == "epd":
        topology = epd_topology(world)
        parallelism = topology
        epp_yaml = EPD_YAML
    fc = args.mode == "fc"

    cfg = NodeConfig(
        model=model_cfg, rank=rank, world_size=world, topology=topology,
        epp_yaml=epp_yaml, device=device, dtype=dtype,
        kv_blocks=None if use_gpu else 2048,
        kv_budget_bytes=int(args.kv_gb * (1 << 30)),
        flow_control=fc,
        fc_bands=[BandConfig(1, ordering="slodeadline"),
                  BandConfig(0, ordering="fcfs"),
                  BandConfig(-1, ordering="fcfs")] if fc else [],
        fc_global_max_items=args.concurrency * 8 if fc else None,
        ttft_slo_ms=args.ttft_slo_ms, kv_cache_dtype=args.kv_dtype,
        mailbox_group=mailbox_group, transfer_group=transfer_group,
        seed=args.seed)
    node = NodeRunner(cfg)

    n_decode = len(node.topology.ranks_with(
        __import__("llm_d_inference_scheduler_amd.datalayer.endpoint",
                   fromlist=["Role"]).Role.DECODE))
    target_inflight = args.concurrency * max(1, n_decode)
    if fc:
        target_inflight *= 2  # 2x overload for the flow-control config

    workload = Workload(args, vocab=model_cfg.vocab_size)
    if rank == 0 and fc:
        node.datastore.put_objective(InferenceObjective(
            "critical", priority=10, ttft_slo_ms=args.ttft_slo_ms))
        node.datastore.put_objective(InferenceObjective(
            "standard", priority=0, ttft_slo_ms=args.ttft_slo_ms))
        node.datastore.put_objective(InferenceObjective(
            "batch", priority=-1, ttft_slo_ms=args.ttft_slo_ms * 5))

    stats = {"completed": 0, "errors": 0, "epp_ms": [], "ttft_ms": [],
             "e2e_ms": []}
    # fc mode: per-priority-tier accounting (BASELINE config 4 is about
    # holding the critical tier's SLO while sheddables are dropped)
    tiers = ["critical", "standard", "batch"]
    tier_stats = {t: {"completed": 0, "shed": 0, "ttft_ms": []}
                  for t in tiers}

    def tier_of(req_id):
        try:
            return tiers[int(req_id.split("-")[-1]) % 3]
        except (ValueError, IndexError):
            return "standard"

    # Pace closed-loop admission to the prefill service rate: one prefill
    # pass is prefill_chunk_tokens (8192) per prompt-running rank, so
    # feeding ~one pass worth of prompts per step keeps every arrival's
    # individual TTFT at ~1 queued pass (well under the SLO) instead of
    # building a cold-start backlog whose tail blows the 2s SLO and then
    # pollutes goodput for the next `max_tokens` steps (slo_ok is frozen
    # per request at first token).
    from llm_d_inference_scheduler_amd.datalayer.endpoint import Role as _R
    n_prompt_ranks = (len(node.topology.ranks_with(_R.PREFILL))
                      or max(1, n_decode))
    ramp = max(1, n_prompt_ranks * 8192 // max(1, args.prompt_len))
    arrival_state = {"next": None}

    def feed(limit=None):
        if rank != 0:
            return
        if args.arrival_rate > 0:
            # open-loop: Poisson arrivals against the wall clock
            now = time.perf_counter()
            if arrival_state["next"] is None:
                arrival_state["next"] = now
            while arrival_state["next"] <= now:
                node.submit(workload.next_request())
                arrival_state["next"] += \
                    workload.rng.expovariate(args.arrival_rate)
            return
        n = 0
        while node.inflight + len(node._arrivals) < target_inflight:
            if limit is not None and n >= limit:
                break
            node.submit(workload.next_request())
            n += 1

    def pace_open_loop():
        """Open-loop runs must track the WALL CLOCK: an idle engine steps
        in ~15 us, so an unpaced loop burns its whole step budget before
        the first Poisson arrival ever lands (found on the fc sweep —
        whole 720-step run finished in 11 ms of wall time). When there is
        no engine work, sleep toward the next scheduled arrival."""
        if rank != 0 or args.arrival_rate <= 0:
            return
        if node.engine.has_work or node.inflight:
            return
        nxt = arrival_state["next"]
        if nxt is not None:
            time.sleep(min(2e-3, max(0.0, nxt - time.perf_counter())))
        else:
            time.sleep(1e-3)

    def drain():
        if rank != 0:
            return
        stats["ttft_ms"].extend(node.drain_ttft_events())
        for c in node.drain_completions():
            if c.error:
                stats["errors"] += 1
                if fc:
                    tier_stats[tier_of(c.request_id)]["shed"] += 1
                continue
            stats["completed"] += 1
            if fc:
                ts = tier_stats[tier_of(c.request_id)]
                ts["completed"] += 1
                if c.usage.ttft_ms is not None:
                    ts["ttft_ms"].append(c.usage.ttft_ms)
            if c.usage.e2e_ms is not None:
                stats["e2e_ms"].append(c.usage.e2e_ms)

    def sync():
        if use_gpu:
            torch.cuda.synchronize()
        if world > 1:
            dist.barrier()
            if use_gpu:
                torch.cuda.synchronize()

    # ---- warmup (ramped admission: the closed-loop cohort arrives over
    # the first half of warmup instead of as one thundering herd whose
    # tail TTFTs blow the SLO before steady state exists) ----
    #
    # --warmup is the MINIMUM number of untimed steps; warmup then continues
    # until steady state so a short driver window (e.g. 20 steps / 5 warmup)
    # reads the steady-state rate instead of the ramp (the
    # 5-warmup window measured 765 tok/s against a 12.5k steady state).
    # Steady state = this rank's decode batch is saturated with no prefill
    # backlog, or its size stopped growing (pool-capacity- or arrival-
    # bound); ranks agree via a MIN all-reduce on the gloo mailbox group
    # every check so the lockstep never diverges. Hard cap bounds runtime.
    from llm_d_inference_scheduler_amd.datalayer.endpoint import Role
    decode_capable = rank in node.topology.ranks_with(Role.DECODE)
    sat_target = 0.95 * min(target_inflight / max(1, n_decode),
                            node.engine.max_decode_batch)
    warmup_cap = max(args.warmup, 600)
    hist = []           # local decode-batch size per warmup step

    def rank_ready() -> bool:
        if not decode_capable:
            return True
        r = len(node.engine.running)
        if r >= sat_target and not node.engine.waiting:
            return True
        # growth stalled below target (e.g. KV-pool-bound): steady anyway
        return (len(hist) >= 24 and r > 0
                and max(hist[-8:]) <= max(hist[-24:-8]))

    w_steps = 0
    while True:
        feed(limit=ramp)
        node.step()
        drain()
        pace_open_loop()
        hist.append(len(node.engine.running))
        w_steps += 1
        if w_steps >= warmup_cap:
            break
        if w_steps >= args.warmup and w_steps % 4 == 0:
            ready = 1.0 if rank_ready() else 0.0
            if world > 1:
                rb = torch.tensor([ready], dtype=torch.float64)
                dist.all_reduce(rb, op=dist.ReduceOp.MIN,
                                group=ctrl_group)
                ready = float(rb[0])
            if ready >= 1.0:
                break
    # TTFT stats intentionally include the ramped warmup cohort: with
    # out=1024 few NEW requests arrive inside a short timed window, and a
    # first-token latency observed during ramp is a real TTFT.

    # ---- timed region: EXACTLY K steps ----
    sync()
    tok0 = node.engine.total_generated
    tok0_slo = node.engine.total_generated_slo
    comp0 = stats["completed"]
    t0 = time.perf_counter()
    for _ in range(args.steps):
        feed()
        node.step()
        drain()
        pace_open_loop()
    sync()
    elapsed = time.perf_counter() - t0
    tokens = node.engine.total_generated - tok0
    tokens_slo = node.engine.total_generated_slo - tok0_slo

    # MAX elapsed over ranks; SUM tokens over ranks
    if world > 1:
        buf = torch.tensor([elapsed], dtype=torch.float64)
        dist.all_reduce(buf, op=dist.ReduceOp.MAX, group=ctrl_group)
        elapsed = float(buf[0])
        tbuf = torch.tensor([tokens, tokens_slo], dtype=torch.float64)
        dist.all_reduce(tbuf, op=dist.ReduceOp.SUM, group=ctrl_group)
        tokens, tokens_slo = float(tbuf[0]), float(tbuf[1])

    if rank == 0:
        completed = stats["completed"] - comp0
        p50_epp = _pctl(list(node.epp_latencies), 50)
        p50_ttft = _pctl(stats["ttft_ms"], 50)
        p99_ttft = _pctl(stats["ttft_ms"], 99)
        goodput = tokens_slo / elapsed
        result = {
            "metric": "routed req/s + p50 EPP latency; P/D goodput "
                      "(tok/s under TTFT SLO) Llama-3-8B",
            "value": round(goodput, 2),
            "unit": "tok/s",
            "n_gpus": world,
            "steps": args.steps,
            "warmup": args.warmup,
            "ms_per_step": round(elapsed * 1e3 / args.steps, 3),
            "higher_is_better": True,
            "scaling": "weak",
            "vs_baseline": None,
            "dtype": "bf16" if use_gpu else "fp32",
            "data": "synthetic shared-prefix prompts, random-init weights",
            "config": {
                "model": model_cfg.name,
                "global_batch": target_inflight,
                "seq_len": args.prompt_len + args.max_tokens,
                "parallelism": parallelism,
                "mode": args.mode,
                "arrival_rate_req_s": args.arrival_rate or None,
                "prompt_len": args.prompt_len,
                "max_tokens": args.max_tokens,
                "kv_cache_dtype": str(node.engine.pool.cache_dtype
                                      ).replace("torch.", ""),
                "ttft_slo_ms": args.ttft_slo_ms,
                "warmup_steps_run": w_steps,
                "routed_req_s": round(completed / elapsed, 2),
                "p50_epp_latency_ms": p50_epp,
                "p50_ttft_ms": p50_ttft,
                "p99_ttft_ms": p99_ttft,
                "total_tok_s": round(tokens / elapsed, 2),
                "errors": stats["errors"],
                **({"tiers": {t: {
                    "completed": v["completed"], "shed": v["shed"],
                    "p50_ttft_ms": _pctl(v["ttft_ms"], 50)}
                    for t, v in tier_stats.items()}} if fc else {}),
            },
        }
        print(json.dumps(result), flush=True)
    node.shutdown()
    if world > 1:
        dist.barrier()
        dist.destroy_process_group()


def layers_main(args):
    """Throughput of a stack of layers, both designs in turn: one JSON line
    whose config holds every measurement."""
    from llm_d_inference_scheduler_amd.engine import layer_bench
    gpu = torch.cuda.is_available() if args.device is None \
        else args.device.startswith("cuda")
    kw = {} if gpu else dict(prompts=2, prompt_len=32, batches=(2,),
                             device="cpu")
    sizes = args.layer_sizes.split(",") if gpu else ["tiny"]
    steps = min(args.steps, 64)
    design = args.layer_design
    rows = layer_bench.run(sizes, design, steps=steps, **kw)
    last = [v for k, v in rows.items() if f"/{design}/" in k][-1]
    print(json.dumps({
        "metric": f"{design.capitalize()} layers: prefill and decode tok/s "
                  "beside Llama layers of equal size",
        "value": last["decode_tok_s"], "unit": "tok/s", "n_gpus": 1,
        "steps": steps, "warmup": 8,
        "ms_per_step": last["decode_ms_per_step"],
        "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "dtype": "bf16" if gpu else "fp32",
        "data": "synthetic prompts, random-init weights",
        "config": {"model": f"{design} layers vs llama layers",
                   "layer_runs": layer_bench.RUNS, "parallelism": "dp1",
                   "results": rows}}), flush=True)


def _pctl(xs, p):
    if not xs:
        return None
    xs = sorted(xs)
    idx = min(len(xs) - 1, int(round(p / 100 * (len(xs) - 1))))
    return round(xs[idx], 3)


if __name__ == "__main__":
    main()
