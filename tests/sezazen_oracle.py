"""Plain, slow float64 implementation of the Sezazen design.

One function per mechanism, whole sequences only, no cache, no batching and
nothing shared with the product path: the tests compare the engine with it.
Tensors are [tokens, features]; a model is (config dict, {name: tensor}).
"""
import math

import torch

F64 = torch.float64


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def relu_squared(z):
    return torch.where(z > 0, z * z, torch.zeros_like(z))


def embedding(table, pos, tokens, scale):
    """Scaled token vectors plus unscaled position vectors."""
    t = torch.as_tensor(list(tokens))
    return table[t] * scale + pos[:len(t)]


def sink_softmax(s, see):
    """Weights of scores s [T, T] where `see` holds, with a score of 0 that
    takes part in the sum only."""
    m = torch.clamp(s.masked_fill(~see, -math.inf).max(-1, keepdim=True)
                    .values, min=0.0)
    e = torch.exp(s - m) * see
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def attention(h, w, m):
    """Causal attention of grouped heads without positions; w: {suffix:
    tensor} of one mixer; m: its sizes."""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w["q"].T).view(T, H, D)
    k = (h @ w["k"].T).view(T, G, D)
    v = (h @ w["v"].T).view(T, G, V)
    see = torch.arange(T)[None, :] <= torch.arange(T)[:, None]
    out = torch.zeros(T, H, V, dtype=h.dtype)
    for head in range(H):
        g = head // (H // G)
        s = (q[:, head] @ k[:, g].T) * m["scale"]
        out[:, head] = sink_softmax(s, see) @ v[:, g]
    return out.reshape(T, H * V) @ w["o"].T


def gated_mlp(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def expert(h, up, down):
    return relu_squared(h @ up.T) @ down.T


def route(h, router, top):
    """-> (chosen experts, their weights), [T, top] each."""
    s = sigmoid(h @ router.T)
    idx = torch.sort(s, dim=-1, descending=True, stable=True).indices[:, :top]
    return idx, torch.gather(s, 1, idx)


def mixture(h, w, m):
    """w: {suffix: tensor} of one feed-forward; every token through its
    chosen experts, the weight on the expert's input."""
    idx, weight = route(h, w["router"], m["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(idx[t].tolist(), weight[t]):
            out[t] += expert((a * h[t])[None], w[f"e{e}.up"],
                             w[f"e{e}.down"])[0]
    if m.get("shared"):
        out = out + expert(h, w["shared.up"], w["shared.down"])
    return out


def layer(x, W, i, entry, eps):
    p = f"l{i}."

    def part(prefix):
        return {k[len(prefix):]: t for k, t in W.items()
                if k.startswith(prefix)}
    x = x + attention(rms_norm(x, W[p + "norm1"], eps), part(p + "mix."),
                      entry["mixer"])
    m = entry.get("mlp")
    if m:
        h = rms_norm(x, W[p + "norm2"], eps)
        w = part(p + "mlp.")
        x = x + (gated_mlp(h, w["gate"], w["up"], w["down"])
                 if m["kind"] == "dense" else mixture(h, w, m))
    return x


def enter_pass(x, x0, W, t):
    """Before the first layer of pass t: mix the stream with the embedding
    output, then add the pass's own vector."""
    return torch.cat([x, x0], -1) @ W["loop.in"].T + W["loop.step"][t]


def forward(cfg, weights, tokens, layers_out=None):
    """tokens -> logits [T, vocab]; layers_out collects the stream."""
    W = {k: t.to(F64) for k, t in weights.items()}
    eps = cfg["norm"]["eps"]
    x0 = embedding(W["embed"], W["pos"], tokens, cfg["embedding"]["scale"])
    x = x0

    def run(x, i):
        x = layer(x, W, i, cfg["layers"][i], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
        return x
    n = len(cfg["layers"])
    loop = cfg.get("loop") or {"start": n, "stop": n, "times": 0}
    for i in range(loop["start"]):
        x = run(x, i)
    for t in range(loop["times"]):
        x = enter_pass(x, x0, W, t)
        for i in range(loop["start"], loop["stop"]):
            x = run(x, i)
    for i in range(loop["stop"], n):
        x = run(x, i)
    return rms_norm(x, W["final.norm"], eps) @ W["embed"].T
