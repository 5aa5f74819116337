"""Small Rururax models for the tests: configurations in the checkpoint's own
keys, random weights, and a folder writer."""
import copy
import math

import torch

import model_files
from model_files import tokens  # noqa: F401

# sizes no kernel has a vector form for: odd groups, unequal dims, two
# windows, a layer without feed-forward, plain rotary
ODD = {
    "architecture": "Rururax", "vocab": 67, "width": 36,
    "embedding": {"scale": 2.5}, "norm": {"eps": 1e-5},
    "layers": [
        {"type": "latent_attention", "mlp": {"kind": "dense", "ff": 22},
         "mixer": {"heads": 3, "dim": 6, "rot_dim": 4, "vdim": 10,
                   "q_rank": 14, "kv_rank": 18, "scale": 0.9,
                   "mask": {"size": 9},
                   "rot": {"dims": 4, "base": 100.0}}},
        {"type": "channel_delta", "mlp": {"kind": "dense", "ff": 26},
         "mixer": {"heads": 6, "kv_heads": 2, "dim": 10, "vdim": 14,
                   "conv": 3}},
        {"type": "latent_attention", "mlp": None,
         "mixer": {"heads": 5, "dim": 8, "rot_dim": 4, "vdim": 7,
                   "q_rank": 9, "kv_rank": 18, "scale": 0.7,
                   "mask": {"size": 21}, "kv_from": 0,
                   "rot": {"dims": 4, "base": 100.0}}},
        {"type": "channel_delta", "mlp": None,
         "mixer": {"heads": 4, "kv_heads": 4, "dim": 7, "vdim": 5,
                   "conv": 1}},
    ]}

# sizes the tiled kernels take, with rotary scaling and shared latents
TILED = {
    "architecture": "Rururax", "vocab": 96, "width": 64,
    "embedding": {"scale": 8.0}, "norm": {"eps": 1e-6},
    "layers": [
        {"type": "channel_delta", "mlp": {"kind": "dense", "ff": 72},
         "mixer": {"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 24,
                   "conv": 4}},
        {"type": "latent_attention", "mlp": {"kind": "dense", "ff": 80},
         "mixer": {"heads": 20, "dim": 16, "rot_dim": 8, "vdim": 24,
                   "q_rank": 40, "kv_rank": 48, "scale": 0.35,
                   "mask": {"size": 37},
                   "rot": {"dims": 8, "base": 5000.0,
                           "scaling": {"factor": 3.0, "original": 64,
                                       "fast": 4.0, "slow": 1.0}}}},
        {"type": "latent_attention", "mlp": {"kind": "dense", "ff": 48},
         "mixer": {"heads": 12, "dim": 24, "rot_dim": 8, "vdim": 16,
                   "q_rank": 24, "kv_rank": 48, "scale": 0.3,
                   "mask": {"size": 70}, "kv_from": 1,
                   "rot": {"dims": 8, "base": 5000.0,
                           "scaling": {"factor": 3.0, "original": 64,
                                       "fast": 4.0, "slow": 1.0}}}},
        {"type": "channel_delta", "mlp": {"kind": "dense", "ff": 72},
         "mixer": {"heads": 2, "kv_heads": 1, "dim": 64, "vdim": 40,
                   "conv": 2}},
    ]}

RANKS = (5, 11)     # inner sizes of the decay and gate projections


def shapes(cfg):
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        for n in ["norm1", "norm1b"] + (["norm2", "norm2b"]
                                        if layer["mlp"] else []):
            out[p + n] = (w,)
        if layer["type"] == "channel_delta":
            H, K, V, ra, rg = m["heads"], m["dim"], m["vdim"], *RANKS
            qk, t = m["kv_heads"] * K, m["conv"]
            mix = {"q": (qk, w), "k": (qk, w), "v": (H * V, w),
                   "q.conv": (qk, t), "k.conv": (qk, t),
                   "v.conv": (H * V, t), "b": (H, w), "A_log": (H,),
                   "norm": (V,), "a1": (ra, w), "a2": (H * K, ra),
                   "dt_bias": (H * K,), "g1": (rg, w), "g2": (H * V, rg),
                   "o": (w, H * V)}
        else:
            H, R = m["heads"], m["kv_rank"]
            mix = {"dq": (m["q_rank"], w), "dq.norm": (m["q_rank"],),
                   "uq": (H * (m["dim"] + m["rot_dim"]), m["q_rank"]),
                   "uk": (H * m["dim"], R), "uv": (H * m["vdim"], R),
                   "o": (w, H * m["vdim"])}
            if "kv_from" not in m:
                mix["dkv"] = (R + m["rot_dim"], w)
                mix["dkv.norm"] = (R,)
        out.update({p + "mix." + k: s for k, s in mix.items()})
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            out[p + "mlp.gate"] = out[p + "mlp.up"] = (ff, w)
            out[p + "mlp.down"] = (w, ff)
    return out


def random_weights(cfg, seed=0):
    """bf16 weights. Scores spread over a few units so that single keys
    matter; decays range from almost none to almost all."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        leaf = name.split(".", 1)[-1]
        if leaf in ("mix.norm", "mix.dq.norm", "mix.dkv.norm"):
            t = 1 + 0.3 * t
        elif len(shape) == 1 and "mix" not in name:
            t = 0.3 * t
        elif leaf == "mix.A_log":
            t = t
        elif leaf == "mix.dt_bias":
            t = 2 * t - 3
        elif leaf.endswith(".conv"):
            t = t / math.sqrt(shape[1])
        else:
            t = t / math.sqrt(shape[-1])
        out[name] = t.bfloat16()
    return out


def write_model(folder, cfg, weights=None, seed=0):
    """-> (folder path, weights)."""
    return model_files.write_model(
        folder, cfg, random_weights(cfg, seed) if weights is None else weights)


def variant(cfg, **changes):
    """Copy of a configuration with mixer fields changed in every layer that
    has them (changes: field=value)."""
    cfg = copy.deepcopy(cfg)
    for layer in cfg["layers"]:
        for k, v in changes.items():
            if k in layer["mixer"]:
                layer["mixer"][k] = v
    return cfg
