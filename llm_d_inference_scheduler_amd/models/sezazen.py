"""Sezazen: configuration reader, tensor names and random init.

Grouped attention without rotation and with a sink in the softmax, dense or
expert feed-forwards, learned positions, and a stretch of layers that runs
several times with the same weights. The computation itself is
`layered.LayeredRunner`; this module only knows the design's configuration
keys and tensor names.
"""
import math
import os
from typing import Any, Callable, Dict, Optional

import torch

from .configs import (ExpertsSpec, FeedForwardSpec, GatedSpec,
                      GroupedAttentionSpec, LayeredConfig, LayerSpec,
                      LoopSpec)

ARCHITECTURE = "Sezazen"


def _feed_forward(i: int, raw: Optional[Dict[str, Any]]
                  ) -> Optional[FeedForwardSpec]:
    if not raw:
        return None
    if raw["kind"] == "dense":
        return GatedSpec(raw["ff"], "silu")
    if raw["kind"] != "moe":
        raise ValueError(f"layer {i}: unknown mlp {raw['kind']!r}")
    shared = raw.get("shared")
    return ExpertsSpec(experts=raw["router"]["experts"],
                       top=raw["router"]["top"], ff=raw["expert"]["ff"],
                       shared_ff=shared["ff"] if shared else None)


def read_config(raw: Dict[str, Any], folder: str) -> LayeredConfig:
    """config.json of a checkpoint folder -> LayeredConfig."""
    layers = []
    for i, entry in enumerate(raw["layers"]):
        if entry["type"] != "attention":
            raise ValueError(f"layer {i}: unknown mixer {entry['type']!r}")
        m = entry["mixer"]
        layers.append(LayerSpec(GroupedAttentionSpec(
            heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
            vdim=m["vdim"], scale=float(m["scale"]), sink=0.0),
            _feed_forward(i, entry.get("mlp"))))
    loop = raw.get("loop")
    return LayeredConfig(
        name=os.path.basename(os.path.normpath(folder)) or "sezazen",
        architecture=ARCHITECTURE, vocab_size=raw["vocab"],
        hidden_size=raw["width"], layers=tuple(layers),
        rms_eps=float(raw["norm"]["eps"]),
        embed_scale=float(raw["embedding"]["scale"]),
        learned_positions=True, max_position=raw["max_positions"],
        loop=LoopSpec(loop["start"], loop["stop"], loop["times"])
        if loop else None, weights_dir=folder)


def tensor_shapes(c: LayeredConfig) -> Dict[str, tuple]:
    """Every tensor of the design, linear weights as [out, in]."""
    w = c.hidden_size
    out = {"embed": (c.vocab_size, w), "pos": (c.max_position, w),
           "final.norm": (w,)}
    if c.loop:
        out["loop.in"] = (w, 2 * w)
        out["loop.step"] = (c.loop.times, w)
    for i, layer in enumerate(c.layers):
        p, m, ff = f"l{i}.", layer.mixer, layer.ff
        out[p + "norm1"] = (w,)
        out[p + "mix.q"] = (m.heads * m.dim, w)
        out[p + "mix.k"] = (m.kv_heads * m.dim, w)
        out[p + "mix.v"] = (m.kv_heads * m.vdim, w)
        out[p + "mix.o"] = (w, m.heads * m.vdim)
        if ff is None:
            continue
        out[p + "norm2"] = (w,)
        if isinstance(ff, GatedSpec):
            out[p + "mlp.gate"] = out[p + "mlp.up"] = (ff.ff, w)
            out[p + "mlp.down"] = (w, ff.ff)
            continue
        out[p + "mlp.router"] = (ff.experts, w)
        inner = {f"e{e}": ff.ff for e in range(ff.experts)}
        if ff.shared_ff:
            inner["shared"] = ff.shared_ff
        for name, n in inner.items():
            out[p + f"mlp.{name}.up"] = (n, w)
            out[p + f"mlp.{name}.down"] = (w, n)
    return out


def random_tensor(name: str, shape: tuple, fill: Callable) -> torch.Tensor:
    """fill(shape, std) draws normal values: norm weights around one,
    vectors that are added to the stream small, projections by fan-in."""
    if name.split(".")[-1] in ("norm1", "norm2", "norm"):
        return fill(shape, 0.1).add_(1.0)
    if name in ("pos", "loop.step"):
        return fill(shape, 0.3)
    if name == "embed":
        return fill(shape, 1.0)
    return fill(shape, 1.0 / math.sqrt(shape[-1]))
