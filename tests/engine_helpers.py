"""Engines of small layer-listed models, fed with given tokens."""
import torch

from llm_d_inference_scheduler_amd.engine import EngineWorker
from llm_d_inference_scheduler_amd.engine.worker import TokenSpan
from llm_d_inference_scheduler_amd.models import registry


def worker(folder, run, blocks=64, slots=4, **kw):
    device, dtype, _ = run
    kw.setdefault("max_model_len", 512)
    return EngineWorker(registry.resolve(folder), device, kv_blocks=blocks,
                        dtype=dtype, state_slots=slots, **kw)


def close(got, want, limit, what=""):
    got, want = got.double().cpu(), want.double()
    err = (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
    assert float(err.mean()) < limit and float(err.max()) < 16 * limit, \
        (what, float(err.mean()), float(err.max()), int(err.argmax()))


def feed(w, rid, toks, cuts, every=True):
    """Run a sequence in portions -> logits of every token (or the last)."""
    rows, at = [], 0
    for n in cuts:
        rows.append(w.forward_spans([TokenSpan(
            rid, toks[at:at + n], list(range(n)) if every else [n - 1])]))
        at += n
    assert at == len(toks)
    return torch.cat(rows)
