"""Torch versions of the `_hip_layered` kernels for CPU tensors (tests, gloo
runs). Same signatures and the same 32-bit inner precision."""
import torch


def _rms(x, w, offset, eps):
    x = x.float()
    return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps) * \
        (w + offset)


def _out(x, wn, offset, eps, f32):
    return (x if wn is None else _rms(x, wn, offset, eps)).to(
        torch.float32 if f32 else torch.bfloat16)


def embed_norm(ids, table, scale, wn, offset, eps, pos, positions):
    x = table[ids].float() * scale
    if pos is not None:
        x += pos[positions.long()]
    return x, _out(x, wn, offset, eps, table.dtype == torch.float32)


def stream_norm(x, y, wb, wn, offset, eps, f32, rows):
    if y is not None:
        x += y if wb is None else _rms(y, wb, offset, eps)
    if rows is not None:
        x += rows.float().view(x.shape[0], -1, x.shape[1]).sum(1)
    return _out(x, wn, offset, eps, f32)


def loop_norm(x, a, b, v, wn, offset, eps, f32):
    x.copy_(a + b + v)
    return _out(x, wn, offset, eps, f32)


def _act(z, act):
    if act == 0:
        return torch.nn.functional.gelu(z, approximate="tanh")
    return torch.nn.functional.silu(z) if act == 1 else z.clamp(min=0) ** 2


def gated_act(gate_up, act):
    g, u = gate_up.float().chunk(2, -1)
    return (_act(g, act) * u).to(gate_up.dtype)


def activate(x, act):
    return _act(x.float(), act).to(x.dtype)


def route(h, w, top):
    z, ids = (h.float() @ w.float().t()).sort(dim=-1, descending=True,
                                              stable=True)
    return ids[:, :top].int(), torch.sigmoid(z[:, :top])


def experts(h, ids, weights, up, down, act, plain):
    top = ids.shape[1]
    out = torch.empty((ids.numel(), h.shape[1]), dtype=h.dtype)
    for e in range(up.shape[0]):
        pairs = (ids.flatten() == e).nonzero().flatten()
        z = h[pairs // top].float() @ up[e].float().t()
        hid = _act(z * weights.flatten()[pairs, None], act).to(h.dtype)
        out[pairs] = (hid.float() @ down[e].float().t()).to(h.dtype)
    return out


def delta_prep(proj, taps, conv_state, row_seq, seq_meta, multi_row, kv_heads,
               heads, dim, vdim, q_scale, unit_eps):
    n_taps, C = taps.shape
    rows = proj.shape[0]
    mixed = torch.empty(rows, C)
    for row0, n, prior, slot in seq_meta.tolist():
        past = conv_state[slot].float() if prior else \
            torch.zeros(n_taps - 1, C)
        seen = torch.cat([past, proj[row0:row0 + n, :C].float()])
        mixed[row0:row0 + n] = sum(
            taps[j] * seen[j:j + n] for j in range(n_taps))
        conv_state[slot] = seen[n:].to(conv_state.dtype)
    mixed = torch.nn.functional.silu(mixed)
    qk = mixed[:, :2 * kv_heads * dim].view(rows, 2, kv_heads, dim)
    qk = qk * torch.rsqrt(qk.pow(2).sum(-1, keepdim=True) + unit_eps)
    return [qk[:, 0] * q_scale, qk[:, 1].contiguous(),
            mixed[:, 2 * kv_heads * dim:].reshape(rows, heads, vdim)]


def delta_step(q, k, v, proj, beta_col, decay, dt_bias, neg_a, gate, norm_w,
               state, seq_meta, n_seqs, out, eps):
    rows, H, V = v.shape
    K = q.shape[2]
    rep = H // q.shape[1]
    q, k = q.repeat_interleave(rep, 1), k.repeat_interleave(rep, 1)
    beta = torch.sigmoid(proj[:, beta_col:beta_col + H].float())
    g = torch.exp(neg_a[None, :, None] * torch.nn.functional.softplus(
        decay.float() + dt_bias).view(rows, H, K))
    gate = torch.sigmoid(gate.float()).view(rows, H, V)
    for row0, n, prior, slot in seq_meta[:n_seqs].tolist():
        S = state[slot].clone() if prior else torch.zeros_like(state[slot])
        for t in range(row0, row0 + n):
            S = S * g[t].unsqueeze(-1)
            u = beta[t].unsqueeze(-1) * (
                v[t] - (S * k[t].unsqueeze(-1)).sum(1))
            S = S + k[t].unsqueeze(-1) * u.unsqueeze(1)
            o = (S * q[t].unsqueeze(-1)).sum(1)
            out[t] = (_rms(o, norm_w, 0.0, eps) * gate[t]).flatten().to(
                out.dtype)
        state[slot] = S


def _rotate(x, cos_sin, positions):
    """x [rows, ..., dims], pairs (2i, 2i + 1)."""
    cs = cos_sin[positions.long()]
    cs = cs.view((x.shape[0],) + (1,) * (x.dim() - 2) + cs.shape[1:])
    u, v = x[..., 0::2].float(), x[..., 1::2].float()
    c, s = cs[..., 0], cs[..., 1]
    return torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2).to(
        x.dtype)


def latent_prep(proj, wq, wkv, cos_sin, positions, slots, cache, eps):
    nq = wq.shape[0]
    if cache is not None:
        nk = wkv.shape[0]
        flat = cache.view(-1, cache.shape[-1])
        flat[slots, :nk] = _rms(proj[:, nq:nq + nk], wkv, 0.0, eps).to(
            cache.dtype)
        flat[slots, nk:] = _rotate(proj[:, nq + nk:], cos_sin, positions)
    return _rms(proj[:, :nq], wq, 0.0, eps).to(proj.dtype)


def rope_part(q, cos_sin, positions, n_abs):
    rot = cos_sin.shape[1] * 2
    D = q.shape[2] - rot
    q[..., D:] = _rotate(q[..., D:], cos_sin, positions)
    return q[:n_abs, :, :D].transpose(0, 1).contiguous()


def heads_to_rows(src, dst):
    n = src.shape[1]
    dst[:n] = src.transpose(0, 1).reshape(n, -1)


def gather_rows(cache, slots):
    return cache.view(-1, cache.shape[-1])[slots]


def _attend(s, v, scale):
    return torch.softmax(s * scale, -1) @ v


def latent_decode(q_lat, q, cache, positions, row_seq, block_tables, window,
                  scale, max_ctx, plain):
    R, W, bs = q_lat.shape[2], cache.shape[2], cache.shape[1]
    flat = cache.view(-1, W)
    out = torch.empty_like(q_lat)
    for i in range(q_lat.shape[1]):
        pos = int(positions[i])
        t = torch.arange(max(0, pos + 1 - window) if window else 0, pos + 1)
        slots = block_tables[int(row_seq[i])].long()[t // bs] * bs + t % bs
        kv = flat[slots].float()
        s = q_lat[:, i].float() @ kv[:, :R].T + \
            q[i, :, q.shape[2] - (W - R):].float() @ kv[:, R:].T
        out[:, i] = _attend(s, kv[:, :R], scale).to(out.dtype)
    return out


def latent_prefill(q, kv, lat, positions, row_seq, base, seq_meta, ctx, tiles,
                   rot, window, scale, out, plain):
    rows, H, Q = q.shape
    D, V = Q - rot, out.shape[1] // H
    k = kv[:, :H * D].view(-1, H, D).float()
    v = kv[:, H * D:].view(-1, H, V).float()
    kr = lat[:, lat.shape[1] - rot:].float()
    for i in range(base, rows):
        pos = int(positions[i])
        row0, first = ctx[int(row_seq[i])].tolist()
        lo = max(0, pos + 1 - window) if window else 0
        a, b = row0 + lo - first, row0 + pos + 1 - first
        s = torch.einsum("hd,thd->ht", q[i, :, :D].float(), k[a:b]) + \
            q[i, :, D:].float() @ kr[a:b].T
        o = torch.einsum("ht,thv->hv", torch.softmax(s * scale, -1), v[a:b])
        out[i] = o.flatten().to(out.dtype)


def store_heads(proj, col, slots, cache, dim):
    G, bs, W = cache.shape[1:]
    k, v = proj[:, col:col + G * W].split([G * dim, G * (W - dim)], 1)
    new = torch.cat([k.unflatten(1, (G, dim)),
                     v.unflatten(1, (G, W - dim))], -1)
    cache[slots // bs, :, slots % bs] = new


def _grouped(proj, cache, positions, row_seq, block_tables, lo, hi, heads,
             dim, scale, sink, out):
    G, bs = cache.shape[1:3]
    for i in range(lo, hi):
        t = torch.arange(int(positions[i]) + 1)
        blocks = block_tables[int(row_seq[i])].long()[t // bs]
        kv = cache[blocks, :, t % bs].float().transpose(0, 1)   # [G, t, W]
        q = proj[i, :heads * dim].float().view(G, heads // G, dim)
        s = q @ kv[..., :dim].transpose(1, 2) * scale
        if sink is not None:
            s = torch.cat([s, torch.full_like(s[..., :1], sink)], -1)
        p = torch.softmax(s, -1)[..., :len(t)]
        out[i] = (p @ kv[..., dim:]).flatten().to(out.dtype)


def grouped_decode(proj, cache, positions, row_seq, block_tables, n, heads,
                   dim, scale, sink, max_ctx, out, plain):
    _grouped(proj, cache, positions, row_seq, block_tables, 0, n, heads, dim,
             scale, sink, out)


def grouped_prefill(proj, cache, positions, row_seq, block_tables, base,
                    seq_meta, tiles, heads, dim, scale, sink, out, plain):
    _grouped(proj, cache, positions, row_seq, block_tables, base,
             proj.shape[0], heads, dim, scale, sink, out)
