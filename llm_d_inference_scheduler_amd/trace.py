"""Trace runner: feeds given token ids through a served model step by step
and writes the logits that are asked for. Nothing is sampled.

    bin/trace_run --model DIR --dtype bfloat16 --out DIR --max-tokens N

Steps come on standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}],
     "end": []}

All entries of a step run as one batch of the engine. `want` lists places
among an entry's tokens; their logits go to OUT/<step>.f32 as 32-bit floats
[wanted, vocab]. Requests under `end` give back their pages and state slots
after the step. Every step is answered with a line `done <step>`.
"""
import argparse
import fcntl
import importlib.util
import json
import os
import subprocess
import sys

PACKAGE = os.path.dirname(os.path.abspath(__file__))
ROOT = os.path.dirname(PACKAGE)
EXTENSION = "_hip_layered"
STATE_SLOTS = 4             # requests live at the same time


def ensure_built() -> None:
    """Compile the model's kernels if this checkout has none yet."""
    name = f"{os.path.basename(PACKAGE)}.{EXTENSION}"

    def built():
        importlib.invalidate_caches()
        return importlib.util.find_spec(name) is not None
    if built():
        return
    os.makedirs(os.path.join(ROOT, "build"), exist_ok=True)
    with open(os.path.join(ROOT, "build", "trace_run.lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        if built():
            return
        env = dict(os.environ, LDS_AMD_ONLY=EXTENSION,
                   PYTORCH_ROCM_ARCH="gfx950")
        subprocess.run([sys.executable, "setup.py", "build_ext", "--inplace"],
                       cwd=ROOT, env=env, stdin=subprocess.DEVNULL,
                       stdout=sys.stderr, check=True)
        if not built():
            raise RuntimeError(f"{EXTENSION} was not built")


def parse_args(argv=None):
    p = argparse.ArgumentParser(
        prog="trace_run", description=__doc__,
        formatter_class=argparse.RawDescriptionHelpFormatter)
    p.add_argument("--model", required=True,
                   help="folder with config.json and model.safetensors")
    p.add_argument("--dtype", choices=["bfloat16", "float32"],
                   default="bfloat16")
    p.add_argument("--out", required=True, help="folder for the logits")
    p.add_argument("--max-tokens", type=int, required=True,
                   help="tokens that live requests hold at most, each "
                        "rounded up to a multiple of 64")
    p.add_argument("--device", default="cuda:0")
    return p.parse_args(argv)


def build_engine(args):
    import torch

    from .engine import EngineWorker
    from .engine.kvcache import BLOCK_SIZE
    from .models import registry
    return EngineWorker(
        registry.resolve(args.model), args.device,
        kv_blocks=-(-args.max_tokens // BLOCK_SIZE),
        dtype=getattr(torch, args.dtype), max_model_len=args.max_tokens,
        state_slots=STATE_SLOTS)


def run_step(engine, step, out_dir) -> None:
    from .engine.worker import TokenSpan
    spans = [TokenSpan(e["id"], e["tokens"], e.get("want", []))
             for e in step["entries"]]
    if spans:
        logits = engine.forward_spans(spans)
        if logits.shape[0]:
            logits.float().cpu().numpy().astype("<f4").tofile(
                os.path.join(out_dir, f"{step['step']}.f32"))
    for rid in step.get("end", []):
        engine.finish_spans(rid)


def main(argv=None) -> int:
    args = parse_args(argv)
    if args.device != "cpu":
        ensure_built()
    engine = build_engine(args)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        run_step(engine, step, args.out)
        print(f"done {step['step']}", flush=True)
    return 0
