"""Prefill and decode throughput of a layer-listed design beside Llama at
equal layer size (`bench.py --mode layers`): random weights, a stack of eight
layer runs, the engine's own steps."""
import sys
import time

import torch

from ..models.configs import LayeredConfig, ModelConfig, _rururax, _sezazen
from .worker import EngineRequest, EngineWorker

VOCAB = 32768
# name -> width, ff, heads
SIZES = {"tiny": (64, 128, 2),              # CPU smoke of the harness
         "2b": (2048, 8192, 16),
         "8b": (4096, 14336, 32),
         "32b": (5120, 25600, 64)}
RUNS = 8
# query and latent rank
RANKS = {"tiny": (32, 32), "2b": (768, 512), "8b": (1536, 512),
         "32b": (1536, 512)}
# experts, top, inner size of an expert and of the shared one: a token uses as
# many feed-forward weights as in Llama's gated MLP
EXPERTS = {"tiny": (8, 4, 32, 64), "2b": (32, 4, 2048, 4096),
           "8b": (32, 4, 3584, 7168), "32b": (32, 4, 6400, 12800)}


def _rururax_stack(size: str) -> LayeredConfig:
    width, ff, heads = SIZES[size]
    q_rank, kv_rank = RANKS[size]
    return _rururax(f"rururax-{size}-layers", VOCAB, width, ff, heads=heads,
                    kv_heads=heads, dim=128, q_rank=q_rank, kv_rank=kv_rank,
                    window=1024, pattern="dddaddds")


def _sezazen_stack(size: str) -> LayeredConfig:
    """Six layers, two of which run twice."""
    width, ff, heads = SIZES[size]
    experts, top, expert_ff, shared_ff = EXPERTS[size]
    return _sezazen(f"sezazen-{size}-layers", VOCAB, width, heads=heads,
                    kv_heads=min(8, heads), dim=128, vdim=128, ff=ff,
                    experts=experts, top=top, expert_ff=expert_ff,
                    shared_ff=shared_ff, pattern="deeeee", loop=(1, 3, 2))


DESIGNS = {"rururax": _rururax_stack, "sezazen": _sezazen_stack}


def configs(size: str, design: str):
    width, ff, heads = SIZES[size]
    return {design: DESIGNS[design](size),
            "llama": ModelConfig(f"llama-{size}-layers", VOCAB, width, ff,
                                 RUNS, heads, min(8, heads), 128)}


def measure(cfg, prompts: int, prompt_len: int, batch: int, steps: int,
            device: str = "cuda:0") -> dict:
    """One engine: time prefill steps of prompts x prompt_len tokens, then
    decode steps of `batch` running requests."""
    gpu = device != "cpu"
    dtype = torch.bfloat16 if gpu else torch.float32
    w = EngineWorker(cfg, device, dtype=dtype,
                     kv_budget_bytes=(24 << 30) if gpu else (64 << 20),
                     prefill_chunk_tokens=prompts * prompt_len,
                     max_decode_batch=batch, prefix_caching=False,
                     max_model_len=prompt_len + steps + 64)
    gen = torch.Generator().manual_seed(0)
    sync = torch.cuda.synchronize if gpu else lambda: None

    def add(n, tag, max_tokens):
        for i in range(n):
            ids = torch.randint(0, VOCAB, (prompt_len,), generator=gen)
            w.add_request(EngineRequest(f"{tag}{i}", ids.tolist(),
                                        max_tokens=max_tokens))

    def prefill(tag):
        add(prompts, tag, 1)
        sync()
        t0 = time.perf_counter()
        w.step()
        sync()
        dt = time.perf_counter() - t0
        while w.has_work:
            w.step()
        return dt
    prefill("warm")
    pre = sorted(prefill(f"p{i}-") for i in range(5))[2]
    add(batch, "d", steps + 40)
    while len(w.running) < batch:
        w.step()
    for _ in range(8):
        w.step()
    sync()
    t0 = time.perf_counter()
    for _ in range(steps):
        w.step()
    sync()
    dec = time.perf_counter() - t0
    return {"prefill_tok_s": round(prompts * prompt_len / pre),
            "prefill_ms": round(pre * 1e3, 3),
            "decode_tok_s": round(batch * steps / dec),
            "decode_ms_per_step": round(dec * 1e3 / steps, 3)}


def run(sizes, design: str = "rururax", prompts: int = 8,
        prompt_len: int = 1024, batches=(32, 256), steps: int = 32,
        device: str = "cuda:0") -> dict:
    out = {}
    for size in sizes:
        for b in batches:
            for name, cfg in configs(size, design).items():  # both in turn
                key = f"{size}/{name}/batch{b}"
                out[key] = measure(cfg, prompts, prompt_len, b, steps, device)
                if device != "cpu":
                    torch.cuda.empty_cache()
                print(key, out[key], file=sys.stderr, flush=True)
    return out
