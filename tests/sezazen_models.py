"""Small Sezazen models for the tests: configurations in the checkpoint's own
keys, random weights, and a folder writer."""
import math

import torch

import model_files
from model_files import tokens  # noqa: F401

CODE = 8        # channels that tell a token's route (random_weights)


def attention(heads, kv_heads, dim, vdim, scale):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "scale": scale}


def moe(experts, top, ff, shared):
    return {"kind": "moe", "router": {"experts": experts, "top": top},
            "expert": {"ff": ff}, "shared": shared and {"ff": shared}}


def entry(mixer, mlp):
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


# sizes no kernel has a vector form for, layers unlike each other, a loop in
# the middle, a layer without feed-forward
ODD = {
    "architecture": "Sezazen", "vocab": 71, "width": 38,
    "embedding": {"scale": 1.75}, "norm": {"eps": 1e-4},
    "max_positions": 300, "loop": {"start": 1, "stop": 3, "times": 2},
    "layers": [
        entry(attention(6, 2, 7, 5, 0.6), moe(5, 2, 11, 13)),
        entry(attention(3, 3, 9, 14, 0.5), {"kind": "dense", "ff": 27}),
        entry(attention(4, 1, 5, 3, 0.8), None),
        entry(attention(5, 1, 6, 6, 0.7), moe(3, 3, 9, None)),
    ]}

# sizes the tiled kernels take; the loop ends the stack
TILED = {
    "architecture": "Sezazen", "vocab": 104, "width": 88,
    "embedding": {"scale": 0.8}, "norm": {"eps": 1e-6},
    "max_positions": 320, "loop": {"start": 2, "stop": 4, "times": 4},
    "layers": [
        entry(attention(6, 2, 24, 40, 0.35), moe(7, 2, 64, 40)),
        entry(attention(20, 1, 16, 72, 0.4), moe(12, 3, 24, 56)),
        entry(attention(4, 4, 72, 24, 0.2), {"kind": "dense", "ff": 120}),
        entry(attention(6, 3, 40, 8, 0.3), moe(4, 1, 128, 16)),
    ]}

# the loop is the whole stack and runs once
ONCE = {
    "architecture": "Sezazen", "vocab": 90, "width": 48,
    "embedding": {"scale": 3.0}, "norm": {"eps": 1e-5},
    "max_positions": 200, "loop": {"start": 0, "stop": 2, "times": 1},
    "layers": [
        entry(attention(2, 2, 8, 16, 0.5), moe(6, 1, 40, 24)),
        entry(attention(8, 2, 16, 8, 0.4), {"kind": "dense", "ff": 56}),
    ]}

# no loop at all
STRAIGHT = {k: v for k, v in ONCE.items() if k != "loop"}


def shapes(cfg):
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "pos": (cfg["max_positions"], w),
           "final.norm": (w,)}
    if cfg.get("loop"):
        out["loop.in"] = (w, 2 * w)
        out["loop.step"] = (cfg["loop"]["times"], w)
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        out[p + "norm1"] = (w,)
        out[p + "mix.q"] = (m["heads"] * m["dim"], w)
        out[p + "mix.k"] = (m["kv_heads"] * m["dim"], w)
        out[p + "mix.v"] = (m["kv_heads"] * m["vdim"], w)
        out[p + "mix.o"] = (w, m["heads"] * m["vdim"])
        if not mlp:
            continue
        out[p + "norm2"] = (w,)
        p += "mlp."
        if mlp["kind"] == "dense":
            out[p + "gate"] = out[p + "up"] = (mlp["ff"], w)
            out[p + "down"] = (w, mlp["ff"])
            continue
        E = mlp["router"]["experts"]
        out[p + "router"] = (E, w)
        for e in [f"e{i}" for i in range(E)] + ["shared"]:
            if e != "shared" or mlp["shared"]:
                ff = mlp["shared" if e == "shared" else "expert"]["ff"]
                out[p + e + ".up"] = (ff, w)
                out[p + e + ".down"] = (w, ff)
    return out


def _clear_router(E, top, codes, g):
    """Router rows on the code channels whose choice is never a close one."""
    best, gap = None, -1.0
    for _ in range(300):
        r = torch.randn(E, CODE, generator=g).bfloat16().float()
        z = (codes @ r.T).sort(-1, descending=True).values
        d = float((z[:, top - 1] - z[:, top]).min()) if top < E else 1.0
        if d > gap:
            best, gap = r, d
    assert gap > 0.2
    return best


def random_weights(cfg, seed=0, clear_routes=True):
    """bf16 weights. With clear_routes a token's experts follow from its id:
    the first channels hold a code that nothing but the norms changes, and
    the routers read only these. Rounding then never changes a choice."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        leaf = name.split(".")[-1]
        if leaf.startswith("norm"):
            t = 1 + 0.2 * t
        elif name in ("pos", "loop.step"):
            t = 0.5 * t
        elif name != "embed":
            t = t / math.sqrt(shape[-1])
            if leaf == "down" and ".e" in name:
                t = 2 * t
        out[name] = t
    if clear_routes:
        codes = torch.randn(9, CODE, generator=g).sign()
        out["embed"][:, :CODE] = codes[torch.arange(cfg["vocab"]) % 9]
        for name, t in out.items():
            if name == "pos" or name == "loop.step":
                t[:, :CODE] = 0
            elif name == "loop.in":
                t[:CODE] = 0
                t[:CODE, :CODE] = torch.eye(CODE)
            elif name.split(".")[-1] in ("o", "down"):
                t[:CODE] = 0
            elif name.endswith("norm2"):
                t[:CODE] = 1
            elif name.endswith("router"):
                i = int(name[1:name.index(".")])
                top = cfg["layers"][i]["mlp"]["router"]["top"]
                t.zero_()
                t[:, :CODE] = _clear_router(t.shape[0], top, codes, g)
    return {k: t.bfloat16() for k, t in out.items()}


def write_model(folder, cfg, weights=None, seed=0):
    """-> (folder path, weights)."""
    return model_files.write_model(
        folder, cfg, random_weights(cfg, seed) if weights is None else weights)
