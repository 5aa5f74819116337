"""Plain, slow float64 implementation of the Rururax design.

One function per mechanism, whole sequences only, no cache, no batching and
nothing shared with the product path: the tests compare the engine with it.
Tensors are [tokens, features]; a model is (config dict, {name: tensor}).
"""
import math

import torch

F64 = torch.float64


def rms(x, eps):
    """x over its root mean square (last axis)."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def zero_centred_norm(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(
        math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z / (1.0 + torch.exp(-z))


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def causal_conv(x, taps):
    """out[t, c] = sum_j taps[c, j] * x[t - (n - 1) + j, c]; zeros before 0."""
    n = taps.shape[1]
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(n):
            s = t - (n - 1) + j
            if s >= 0:
                out[t] += taps[:, j] * x[s]
    return out


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_scan(q, k, v, g, beta, state=None):
    """q, k, g: [T, H, K]; v: [T, H, V]; beta: [T, H]. Token by token:
    decay the rows of S, write beta (v - S'k) along k, then read with q."""
    T, H, K = q.shape
    S = torch.zeros(H, K, v.shape[2], dtype=q.dtype) if state is None \
        else state.clone()
    out = torch.zeros_like(v)
    for t in range(T):
        for h in range(H):
            S[h] = g[t, h][:, None] * S[h]
            u = beta[t, h] * (v[t, h] - S[h].T @ k[t, h])
            S[h] = S[h] + torch.outer(k[t, h], u)
            out[t, h] = S[h].T @ q[t, h]
    return out, S


def channel_delta(h, w, m, eps):
    """w: {suffix: tensor} of one mixer; m: its sizes."""
    T = h.shape[0]
    H, KH, K, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]

    def lane(name):
        return silu(causal_conv(h @ w[name].T, w[name + ".conv"]))
    q = unit(lane("q").view(T, KH, K)) * K ** -0.5
    k = unit(lane("k").view(T, KH, K))
    v = lane("v").view(T, H, V)
    src = torch.arange(H) // (H // KH)
    beta = sigmoid(h @ w["b"].T)
    raw = ((h @ w["a1"].T) @ w["a2"].T + w["dt_bias"]).view(T, H, K)
    g = torch.exp(-torch.exp(w["A_log"])[None, :, None] * softplus(raw))
    o, _ = delta_scan(q[:, src], k[:, src], v, g, beta)
    gate = sigmoid((h @ w["g1"].T) @ w["g2"].T).view(T, H, V)
    o = rms(o, eps) * w["norm"] * gate
    return o.reshape(T, H * V) @ w["o"].T


def yarn_frequencies(rot):
    """-> (frequencies [dims/2], factor on cos and sin)."""
    dims, base = rot["dims"], rot["base"]
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)],
                     dtype=F64)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def edge(turns):
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) / \
            (2 * math.log(base))
    lo = max(math.floor(edge(sc["fast"])), 0)
    hi = min(math.ceil(edge(sc["slow"])), dims - 1)
    ramp = torch.tensor([min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
                         for i in range(dims // 2)], dtype=F64)
    return (f / sc["factor"]) * ramp + f * (1 - ramp), \
        0.1 * math.log(sc["factor"]) + 1.0


def rotate_pairs(x, rot):
    """Interleaved rotation of x [T, ..., dims]; row t is position t."""
    f, amp = yarn_frequencies(rot)
    a = torch.arange(x.shape[0], dtype=F64)[:, None] * f
    a = a.view((x.shape[0],) + (1,) * (x.dim() - 2) + (-1,))
    c, s = torch.cos(a) * amp, torch.sin(a) * amp
    u, v = x[..., 0::2], x[..., 1::2]
    return torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2)


def latents(h, w, m, eps):
    """-> (c [T, kv_rank], rotated key part [T, rot_dim])."""
    both = h @ w["dkv"].T
    c = rms(both[:, :m["kv_rank"]], eps) * w["dkv.norm"]
    return c, rotate_pairs(both[:, m["kv_rank"]:], m["rot"])


def latent_attention(h, w, m, eps, shared=None):
    """shared: another layer's (c, key part), for a mixer without its own.
    -> (output, the pair it used)."""
    T = h.shape[0]
    H, D, R, V = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    cq = rms(h @ w["dq"].T, eps) * w["dq.norm"]
    q = (cq @ w["uq"].T).view(T, H, D + R)
    qn, qr = q[..., :D], rotate_pairs(q[..., D:], m["rot"])
    c, kr = latents(h, w, m, eps) if shared is None else shared
    kn = (c @ w["uk"].T).view(T, H, D)
    v = (c @ w["uv"].T).view(T, H, V)
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    see = j <= i
    if m.get("mask"):
        see &= (i - j) < m["mask"]["size"]
    out = torch.zeros(T, H, V, dtype=h.dtype)
    for hd in range(H):
        s = (qn[:, hd] @ kn[:, hd].T + qr[:, hd] @ kr.T) * m["scale"]
        s = s.masked_fill(~see, -math.inf)
        p = torch.exp(s - s.max(-1, keepdim=True).values)
        out[:, hd] = (p / p.sum(-1, keepdim=True)) @ v[:, hd]
    return out.reshape(T, H * V) @ w["o"].T, (c, kr)


def gated_mlp(h, gate, up, down):
    return (gelu_tanh(h @ gate.T) * (h @ up.T)) @ down.T


def forward(cfg, weights, tokens, layers_out=None):
    """tokens -> logits [T, vocab]; layers_out collects the stream."""
    W = {k: t.to(F64) for k, t in weights.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(list(tokens))] * cfg["embedding"]["scale"]
    kept = {}
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        m = layer["mixer"]
        mix = {k[len(p) + 4:]: t for k, t in W.items()
               if k.startswith(p + "mix.")}
        h = zero_centred_norm(x, W[p + "norm1"], eps)
        if layer["type"] == "channel_delta":
            y = channel_delta(h, mix, m, eps)
        else:
            src = m.get("kv_from")
            y, kept[i] = latent_attention(
                h, mix, m, eps, kept[src] if src is not None else None)
        x = x + zero_centred_norm(y, W[p + "norm1b"], eps)
        if layer.get("mlp"):
            h = zero_centred_norm(x, W[p + "norm2"], eps)
            y = gated_mlp(h, W[p + "mlp.gate"], W[p + "mlp.up"],
                          W[p + "mlp.down"])
            x = x + zero_centred_norm(y, W[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return zero_centred_norm(x, W["final.norm"], eps) @ W["embed"].T
