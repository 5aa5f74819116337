"""Rururax: configuration reader, tensor names and random init.

A stack of gated-delta-rule layers with per-channel decay and latent
attention layers (some of which attend to an earlier layer's cached
latents), every sublayer normed before and after, tied embeddings. The
computation itself is `layered.LayeredRunner`; this module only knows the
design's configuration keys and tensor names.
"""
import math
import os
from typing import Any, Callable, Dict

import torch

from .checkpoint import read_safetensors
from .configs import (ChannelDeltaSpec, GatedSpec, LatentAttentionSpec,
                      LayeredConfig, LayerSpec, RotarySpec)

ARCHITECTURE = "Rururax"


def _rotary(raw: Dict[str, Any]) -> RotarySpec:
    s = raw.get("scaling")
    if not s:
        return RotarySpec(dims=raw["dims"], base=float(raw["base"]))
    return RotarySpec(dims=raw["dims"], base=float(raw["base"]),
                      factor=float(s["factor"]),
                      original=float(s["original"]),
                      fast=float(s["fast"]), slow=float(s["slow"]))


def read_config(raw: Dict[str, Any], folder: str) -> LayeredConfig:
    """config.json of a checkpoint folder -> LayeredConfig. The inner sizes
    of the decay and gate projections stand in tensor shapes only."""
    shapes = {k: tuple(t.shape) for k, t in read_safetensors(
        os.path.join(folder, "model.safetensors")).items()}
    layers = []
    for i, entry in enumerate(raw["layers"]):
        m, kind = entry["mixer"], entry["type"]
        if kind == "channel_delta":
            mixer = ChannelDeltaSpec(
                heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
                vdim=m["vdim"], conv=m["conv"],
                decay_rank=shapes[f"l{i}.mix.a1"][0],
                gate_rank=shapes[f"l{i}.mix.g1"][0])
        elif kind == "latent_attention":
            mask = m.get("mask")
            mixer = LatentAttentionSpec(
                heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"],
                vdim=m["vdim"], q_rank=m["q_rank"], kv_rank=m["kv_rank"],
                scale=float(m["scale"]), rot=_rotary(m["rot"]),
                window=mask["size"] if mask else None,
                kv_from=m.get("kv_from"))
        else:
            raise ValueError(f"layer {i}: unknown mixer {kind!r}")
        mlp = entry.get("mlp")
        if mlp and mlp["kind"] != "dense":
            raise ValueError(f"layer {i}: unknown mlp {mlp['kind']!r}")
        layers.append(LayerSpec(mixer, GatedSpec(mlp["ff"]) if mlp else None))
    return LayeredConfig(
        name=os.path.basename(os.path.normpath(folder)) or "rururax",
        architecture=ARCHITECTURE, vocab_size=raw["vocab"],
        hidden_size=raw["width"], layers=tuple(layers),
        rms_eps=float(raw["norm"]["eps"]), norm_offset=1.0, post_norms=True,
        embed_scale=float(raw["embedding"]["scale"]), weights_dir=folder)


def tensor_shapes(c: LayeredConfig) -> Dict[str, tuple]:
    """Every tensor of the design, linear weights as [out, in]."""
    w = c.hidden_size
    out = {"embed": (c.vocab_size, w), "final.norm": (w,)}
    for i, layer in enumerate(c.layers):
        p, m = f"l{i}.", layer.mixer
        for norm in ("norm1", "norm1b") + (("norm2", "norm2b")
                                           if layer.ff else ()):
            out[p + norm] = (w,)
        if isinstance(m, ChannelDeltaSpec):
            qk, v, gv = m.kv_heads * m.dim, m.heads * m.vdim, m.heads * m.dim
            mix = {"q": (qk, w), "q.conv": (qk, m.conv),
                   "k": (qk, w), "k.conv": (qk, m.conv),
                   "v": (v, w), "v.conv": (v, m.conv),
                   "b": (m.heads, w), "A_log": (m.heads,),
                   "norm": (m.vdim,), "a1": (m.decay_rank, w),
                   "a2": (gv, m.decay_rank), "dt_bias": (gv,),
                   "g1": (m.gate_rank, w), "g2": (v, m.gate_rank),
                   "o": (w, v)}
        else:
            mix = {"dq": (m.q_rank, w), "dq.norm": (m.q_rank,),
                   "uq": (m.heads * (m.dim + m.rot_dim), m.q_rank),
                   "uk": (m.heads * m.dim, m.kv_rank),
                   "uv": (m.heads * m.vdim, m.kv_rank),
                   "o": (w, m.heads * m.vdim)}
            if m.kv_from is None:
                mix["dkv"] = (m.kv_rank + m.rot_dim, w)
                mix["dkv.norm"] = (m.kv_rank,)
        for k, shape in mix.items():
            out[p + "mix." + k] = shape
        if layer.ff:
            out[p + "mlp.gate"] = out[p + "mlp.up"] = (layer.ff.ff, w)
            out[p + "mlp.down"] = (w, layer.ff.ff)
    return out


def random_tensor(name: str, shape: tuple, fill: Callable) -> torch.Tensor:
    """fill(shape, std) draws normal values. Norm weights stored around one
    or zero, decays between slow and fast, projections by fan-in."""
    leaf = name.split(".", 1)[-1]
    if leaf in ("mix.norm", "mix.dq.norm", "mix.dkv.norm"):
        return fill(shape, 0.1).add_(1.0)
    if leaf.startswith("norm") or name == "final.norm":
        return fill(shape, 0.1)
    if leaf == "mix.A_log":
        return fill(shape, 0.7)
    if leaf == "mix.dt_bias":
        return fill(shape, 1.0).sub_(3.0)
    return fill(shape, 1.0 / math.sqrt(shape[-1]))
