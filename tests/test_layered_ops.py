"""The layer-listed designs' ops one by one against the plain oracle: the CPU
versions everywhere, the HIP kernels in both precisions on a GPU."""
import math

import pytest
import torch

import rururax_oracle as oracle
from llm_d_inference_scheduler_amd.models import layered, rotary
from llm_d_inference_scheduler_amd.models.configs import RotarySpec
from llm_d_inference_scheduler_amd.ops import layered as ops

GPU = pytest.mark.gpu
RUNS = [pytest.param(("cpu", torch.float32), id="cpu-f32"),
        pytest.param(("cuda:0", torch.float32), id="gpu-f32", marks=GPU),
        pytest.param(("cuda:0", torch.bfloat16), id="gpu-bf16", marks=GPU)]
F64 = torch.float64


def rnd(*shape, seed=0, scale=1.0):
    g = torch.Generator().manual_seed(seed + 7 * len(shape))
    return torch.randn(shape, generator=g) * scale


def put(t, run, dtype=None):
    return t.to(dtype or run[1]).contiguous().to(run[0])


def f64(t):
    return t.double().cpu()


def close(got, want, run, f32=2e-6, bf16=8e-3):
    """Largest error relative to the largest value."""
    tol = bf16 if run[1] == torch.bfloat16 else f32
    got, want = f64(got), want.double()
    assert got.shape == want.shape
    err = (got - want).abs().max() / want.abs().max().clamp(min=1e-30)
    assert float(err) < tol, float(err)


def meta(seqs, run):
    """[(rows, prior, slot)] -> seq_meta, row_seq."""
    out, rows = [], []
    row = 0
    for i, (n, prior, slot) in enumerate(seqs):
        out.append((row, n, prior, slot))
        rows += [i] * n
        row += n
    dev = run[0]
    return (torch.tensor(out, dtype=torch.int32, device=dev),
            torch.tensor(rows, dtype=torch.int32, device=dev))


@pytest.mark.parametrize("run", RUNS)
class TestStream:
    @pytest.mark.parametrize("width", [36, 64, 1000, 4096, 9000])
    def test_norm_and_residual(self, run, width):
        x, y = rnd(5, width), rnd(5, width, seed=1, scale=3)
        wb, wn = rnd(width, seed=2), rnd(width, seed=3)
        xd, yd = x.clone().to(run[0]), put(y, run)
        h = ops.stream_norm(xd, yd, wb.to(run[0]), wn.to(run[0]), 1.0, 1e-3,
                            run[1])
        want = x.double() + oracle.zero_centred_norm(f64(yd), wb.double(),
                                                     1e-3)
        assert (f64(xd) - want).abs().max() < 3e-5      # stays 32-bit
        close(h, oracle.zero_centred_norm(want, wn.double(), 1e-3), run)
        # plain weights, no residual
        h = ops.stream_norm(xd, None, None, wn.to(run[0]), 0.0, 1e-3, run[1])
        close(h, oracle.rms(f64(xd), 1e-3) * wn.double(), run)

    @pytest.mark.parametrize("width", [36, 64])
    def test_embedding(self, run, width):
        table = put(rnd(11, width), run)
        ids = torch.tensor([3, 0, 10, 3], device=run[0])
        wn = rnd(width, seed=3)
        x, h = ops.embed_norm(ids, table, 13.5, wn.to(run[0]), 1.0, 1e-6)
        want = f64(table)[ids.cpu()] * 13.5
        assert x.dtype == torch.float32
        assert (f64(x) - want).abs().max() < 1e-5
        close(h, oracle.zero_centred_norm(want, wn.double(), 1e-6), run)

    @pytest.mark.parametrize("size", [22, 64])
    def test_gelu(self, run, size):
        gu = put(rnd(7, 2 * size, scale=4), run)
        gu[0, 0], gu[0, 1] = 60.0, -60.0
        want = oracle.gelu_tanh(f64(gu)[:, :size]) * f64(gu)[:, size:]
        close(ops.gated_act(gu, "gelu_tanh"), want, run)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("KH,H,K,V,taps", [
    (2, 4, 10, 14, 3), (2, 2, 16, 24, 4), (1, 3, 128, 128, 4),
    (3, 3, 32, 8, 2), (2, 2, 8, 16, 1), (1, 1, 24, 40, 5), (1, 2, 8, 8, 4)])
class TestDeltaPrep:
    def test_convolutions_and_unit_norms(self, run, KH, H, K, V, taps):
        """Portions of a sequence (also shorter than the taps) against the
        whole one; slots of other sequences stay as they are."""
        C = 2 * KH * K + H * V
        total = 23
        proj = put(rnd(total, C + 8), run)
        w = rnd(C, taps, seed=1)
        state = put(rnd(3, taps - 1, C, seed=2), run)
        before = state.clone()
        mixed = oracle.silu(oracle.causal_conv(f64(proj)[:, :C], w.double()))
        q = oracle.unit(mixed[:, :KH * K].view(total, KH, K)) * 0.3
        k = oracle.unit(mixed[:, KH * K:2 * KH * K].view(total, KH, K))
        v = mixed[:, 2 * KH * K:].view(total, H, V)
        wt = w.t().contiguous().to(run[0])
        at = 0
        for n in (2, 1, 1, 5, 1, 13):
            m, rows = meta([(n, at, 1)], run)
            got = ops.delta_prep(proj[at:at + n].contiguous(), wt, state,
                                 rows, m, n > 1, KH, H, K, V, 0.3, 1e-6)
            for a, b in zip(got, (q, k, v)):
                assert a.dtype == torch.float32
                close(a, b[at:at + n], ("", torch.float32), f32=1e-5)
            at += n
        assert torch.equal(state[0], before[0])
        assert torch.equal(state[2], before[2])
        if taps > 1:
            assert torch.equal(state[1], proj[total - taps + 1:, :C])

    def test_batch(self, run, KH, H, K, V, taps):
        C = 2 * KH * K + H * V
        seqs = [(1, 0, 2), (6, 0, 0), (1, 4, 1), (40, 3, 3)]
        rows = sum(s[0] for s in seqs)
        proj = put(rnd(rows, C, seed=5), run)
        state = put(rnd(4, taps - 1, C, seed=6), run)
        w = rnd(C, taps, seed=7)
        m, rs = meta(seqs, run)
        past = f64(state).clone()
        got = ops.delta_prep(proj, w.t().contiguous().to(run[0]), state, rs,
                             m, True, KH, H, K, V, 1.0, 1e-6)
        row = 0
        for n, prior, slot in seqs:
            old = past[slot] if prior else torch.zeros_like(past[slot])
            seen = torch.cat([old, f64(proj)[row:row + n]])
            mixed = oracle.silu(oracle.causal_conv(seen, w.double()))
            close(got[2][row:row + n],
                  mixed[taps - 1:, 2 * KH * K:].reshape(n, H, V),
                  ("", torch.float32), f32=1e-5)
            assert torch.equal(f64(state[slot]), seen[n:])
            row += n


def delta_case(run, seqs, KH, H, K, V, decay_shift, seed=0):
    rows = sum(s[0] for s in seqs)
    dev = run[0]
    d = {"q": oracle.unit(rnd(rows, KH, K, seed=seed)) * K ** -0.5,
         "k": oracle.unit(rnd(rows, KH, K, seed=seed + 1)),
         "v": rnd(rows, H, V, seed=seed + 2)}
    # repeated keys: later writes have to correct earlier ones
    d["k"][rows // 2:] = d["k"][:rows - rows // 2]
    d = {k: t.float().contiguous().to(dev) for k, t in d.items()}
    d["proj"] = put(rnd(rows, 5 + H + 2, seed=seed + 3), run)
    d["decay"] = put(rnd(rows, H * K, seed=seed + 4), run)
    d["bias"] = (rnd(H * K, seed=seed + 5) * 2 + decay_shift).to(dev)
    d["neg_a"] = -torch.exp(rnd(H, seed=seed + 6)).to(dev)
    d["gate"] = put(rnd(rows, H * V, seed=seed + 7), run)
    d["norm"] = (1 + rnd(V, seed=seed + 8) * 0.2).to(dev)
    d["state"] = rnd(5, H, K, V, seed=seed + 9).to(dev)
    return d


def delta_oracle(d, seqs, eps):
    H, K = d["state"].shape[1:3]
    KH = d["q"].shape[1]
    V = d["v"].shape[2]
    src = torch.arange(H) // (H // KH)
    beta = oracle.sigmoid(f64(d["proj"])[:, 5:5 + H])
    g = torch.exp(f64(d["neg_a"])[None, :, None] * oracle.softplus(
        f64(d["decay"]) + f64(d["bias"])).view(-1, H, K))
    outs, raw, states, row = [], [], {}, 0
    for n, prior, slot in seqs:
        s = slice(row, row + n)
        S0 = f64(d["state"])[slot] if prior else None
        o, S = oracle.delta_scan(f64(d["q"])[s][:, src], f64(d["k"])[s][:, src],
                                 f64(d["v"])[s], g[s], beta[s], S0)
        raw.append(o)
        o = oracle.rms(o, eps) * f64(d["norm"]) * oracle.sigmoid(
            f64(d["gate"])[s].view(n, H, V))
        outs.append(o.reshape(n, H * V))
        states[slot] = S
        row += n
    return torch.cat(outs), torch.cat(raw), states


DECAYS = [-9.0, -2.0, 4.0]      # keeps all; some; forgets at once
SIZES = [(2, 4, 10, 14), (2, 2, 16, 24), (1, 2, 32, 32), (1, 1, 64, 40),
         (1, 2, 128, 128), (2, 2, 7, 5), (1, 1, 100, 36)]


@pytest.mark.parametrize("shift", DECAYS)
@pytest.mark.parametrize("KH,H,K,V", SIZES + [(1, 1, 200, 20)])
class TestDelta:
    @pytest.mark.parametrize("run", RUNS)
    def test_steps(self, run, KH, H, K, V, shift):
        seqs = [(1, 3, 2), (1, 0, 4), (7, 0, 1), (5, 9, 0)]
        d = delta_case(run, seqs, KH, H, K, V, shift)
        m, _ = meta(seqs, run)
        want, _, states = delta_oracle(d, seqs, 1e-5)
        idle = d["state"][3].clone()
        out = torch.zeros(14, H * V, dtype=run[1], device=run[0])
        ops.delta_step(d["q"], d["k"], d["v"], d["proj"], 5, d["decay"],
                       d["bias"], d["neg_a"], d["gate"], d["norm"],
                       d["state"], m, 4, out, 1e-5)
        close(out, want, run, f32=2e-5)
        for slot, S in states.items():
            close(d["state"][slot], S, ("", torch.float32), f32=1e-5)
        assert torch.equal(d["state"][3], idle)

    @GPU
    @pytest.mark.parametrize("run", RUNS[1:])
    @pytest.mark.parametrize("per_group", [1, 3, 64])
    def test_chunks(self, run, KH, H, K, V, shift, per_group):
        """Portions around the chunk and block sizes, in one group and in
        several, from a stored and from an empty state."""
        work = ops.delta_chunk_work(K, V, torch.device("cuda"))
        if not work:
            assert K > 128
            return
        seqs = [(64, 0, 2), (9, 5, 4), (130, 0, 1), (81, 3, 0), (16, 1, 3)]
        d = delta_case(run, seqs, KH, H, K, V, shift, seed=50)
        want, raw, states = delta_oracle(d, seqs, 1e-5)
        row, long = 0, []
        for i, (n, prior, slot) in enumerate(seqs):
            long.append(layered.Portion(i, row, n, prior, [], slot))
            row += n
        o = torch.zeros(row, H * V, device=run[0])
        groups = layered.chunk_groups(long, per_group,
                                      torch.device(run[0]))
        ws = torch.full((work * H * per_group,), float("nan"), device=run[0])
        for g in groups:
            ops.delta_chunk(d["q"], d["k"], d["v"], d["proj"], 5, d["decay"],
                            d["bias"], d["neg_a"], d["state"], g, ws, o)
        close(o.view(row, H, V), raw, ("", torch.float32), f32=3e-5)
        for slot, S in states.items():
            close(d["state"][slot], S, ("", torch.float32), f32=3e-5)
        out = torch.zeros(row, H * V, dtype=run[1], device=run[0])
        ops.delta_gate(o, d["gate"], d["norm"], out, 64, 1e-5)
        assert not out[:64].any()
        # the norm magnifies rows whose output is almost nothing
        loud = raw.pow(2).mean(-1).sqrt() > 1e-3 * raw.abs().max()
        got, ref = out.view(row, H, V)[64:], want.view(row, H, V)[64:]
        close(got[loud[64:].to(run[0])], ref[loud[64:]], run, f32=3e-3)


class TestRotary:
    @pytest.mark.parametrize("scaling", [
        None, {"factor": 4.0, "original": 64, "fast": 32.0, "slow": 1.0},
        {"factor": 2.5, "original": 4096, "fast": 8.0, "slow": 2.0},
        {"factor": 16.0, "original": 32, "fast": 1.0, "slow": 0.25}])
    @pytest.mark.parametrize("dims,base", [(4, 100.0), (32, 25000.0),
                                           (64, 1e6)])
    def test_tables(self, dims, base, scaling):
        raw = {"dims": dims, "base": base}
        spec = RotarySpec(dims, base)
        if scaling:
            raw["scaling"] = scaling
            spec = RotarySpec(dims, base, True, **scaling)
        f, amp = oracle.yarn_frequencies(raw)
        got, gamp = rotary.frequencies(spec)
        assert torch.allclose(f, got, rtol=1e-12) and amp == gamp
        x = rnd(40, dims).double()
        t = rotary.table(spec, 40, "cpu").double()
        u, v = x[:, 0::2], x[:, 1::2]
        y = torch.stack([u * t[..., 0] - v * t[..., 1],
                         v * t[..., 0] + u * t[..., 1]], -1).flatten(1)
        assert (y - oracle.rotate_pairs(x, raw)).abs().max() < 1e-5


@pytest.mark.parametrize("run", RUNS)
class TestLatentPrep:
    @pytest.mark.parametrize("q_rank,kv_rank,rot", [(14, 18, 4), (40, 48, 8),
                                                    (300, 512, 64)])
    def test_norms_rotation_and_pages(self, run, q_rank, kv_rank, rot):
        raw = {"dims": rot, "base": 500.0,
               "scaling": {"factor": 2.0, "original": 16, "fast": 4.0,
                           "slow": 1.0}}
        spec = RotarySpec(rot, 500.0, True, **raw["scaling"])
        table = rotary.table(spec, 64, run[0])
        proj = put(rnd(9, q_rank + kv_rank + rot), run)
        wq, wkv = rnd(q_rank, seed=1), rnd(kv_rank, seed=2)
        pos = torch.tensor([0, 1, 2, 31, 32, 63, 5, 5, 17], dtype=torch.int32)
        slots = torch.tensor([16, 3, 47, 0, 22, 31, 32, 15, 40])
        cache = put(rnd(3, 16, kv_rank + rot, seed=3), run)
        keep = cache.clone()
        cq = ops.latent_prep(proj, wq.to(run[0]), wkv.to(run[0]), table,
                             pos.to(run[0]), slots.to(run[0]), cache, 1e-4)
        p = f64(proj)
        close(cq, oracle.rms(p[:, :q_rank], 1e-4) * wq.double(), run)
        rows = f64(cache).view(48, -1)
        close(rows[slots, :kv_rank],
              oracle.rms(p[:, q_rank:q_rank + kv_rank], 1e-4) * wkv.double(),
              run)
        far = torch.zeros(64, 9, rot, dtype=F64)
        far[:] = p[None, :, q_rank + kv_rank:]
        turned = oracle.rotate_pairs(far, raw)[pos.long(), torch.arange(9)]
        close(rows[slots, kv_rank:], turned, run)
        idle = torch.ones(48, dtype=torch.bool)
        idle[slots] = False
        assert torch.equal(rows[idle], f64(keep).view(48, -1)[idle])
        # a layer on another one's latents only norms its queries
        again = ops.latent_prep(proj[:, :q_rank].contiguous(), wq.to(run[0]),
                                None, table, pos.to(run[0]),
                                slots.to(run[0]), None, 1e-4)
        assert torch.equal(again, cq)
        # queries: rotated part in place, plain part by head
        q = put(rnd(9, 3, 6 + rot, seed=4), run)
        old = f64(q)
        plain = ops.rope_part(q, table, pos.to(run[0]), 4)
        close(plain, old[:4, :, :6].transpose(0, 1), run)
        assert torch.equal(f64(q)[..., :6], old[..., :6])
        far = torch.zeros(64, 9, 3, rot, dtype=F64)
        far[:] = old[None, ..., 6:]
        close(q[..., 6:],
              oracle.rotate_pairs(far, raw)[pos.long(), torch.arange(9)], run)
        # and rows back out of the pages
        assert torch.equal(ops.gather_rows(cache, slots.to(run[0])),
                           cache.view(48, -1)[slots.to(run[0])])
        dst = torch.zeros(6, 18, dtype=run[1], device=run[0])
        ops.heads_to_rows(plain, dst.view(6, 18))
        assert torch.equal(dst[:4].view(4, 3, 6), q[:4, :, :6])
        assert not dst[4:].any()


def stand_out(keys, pos, window, big):
    """For every row a direction on which one key stands out: in turn the
    oldest key it sees, the one just before that, itself, the next one and
    the very first."""
    rows = []
    n = keys.shape[0]
    for i, p in enumerate(pos):
        w = window or p + 1
        j = (p - w + 1, p - w, p, p + 1, 0)[i % 5]
        rows.append(keys[min(max(j, 0), n - 1)] * big)
    return torch.stack(rows)


LATENT = [  # H, D, rot, V, R
    (3, 6, 4, 10, 18), (20, 16, 8, 24, 48), (5, 64, 32, 64, 64),
    (33, 128, 64, 128, 512), (16, 64, 64, 64, 128), (8, 32, 32, 64, 256),
    (2, 160, 32, 136, 96)]


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("H,D,rot,V,R", LATENT)
class TestLatentAttention:
    def pages(self, run, R, rot, lens):
        """Latents of several sequences in shuffled pages."""
        bs = 16
        need = [-(-n // bs) for n in lens]
        order = torch.randperm(sum(need) + 2,
                               generator=torch.Generator().manual_seed(3))
        bt = torch.zeros(len(lens), max(need), dtype=torch.int32)
        cache = put(rnd(sum(need) + 2, bs, R + rot, seed=9, scale=30), run)
        lat, at = [], 0
        for s, n in enumerate(lens):
            blocks = order[at:at + need[s]]
            at += need[s]
            bt[s, :need[s]] = blocks.int()
            x = rnd(n, R + rot, seed=20 + s)
            x = x / x.norm(dim=-1, keepdim=True) * math.sqrt(R + rot) / 4
            x = put(x, run)
            slots = blocks[torch.arange(n) // bs] * bs + torch.arange(n) % bs
            cache.view(-1, R + rot)[slots.to(run[0])] = x
            lat.append((x, slots))
        return cache, bt.to(run[0]), lat

    @pytest.mark.parametrize("window", [None, 1, 16, 17, 100])
    def test_decode(self, run, H, D, rot, V, R, window):
        lens = [130, 1, 16, 300]
        cache, bt, lat = self.pages(run, R, rot, lens)
        rows = [(0, 129), (1, 0), (2, 15), (2, 14), (3, 299), (3, 298),
                (3, 160), (0, 64), (0, 100), (3, 0)]
        scale = 0.5
        q = torch.stack([stand_out(f64(lat[s][0]), [p] * 5, window, 3.0)[
            i % 5] for i, (s, p) in enumerate(rows)])
        q = q[:, None] * (0.5 + torch.rand(
            10, H, 1, generator=torch.Generator().manual_seed(1)).double())
        q_lat = put(q[..., :R].transpose(0, 1), run)
        full = put(torch.cat([rnd(10, H, D, seed=2).double(), q[..., R:]],
                             -1), run)
        pos = torch.tensor([p for _, p in rows], dtype=torch.int32,
                           device=run[0])
        seq = torch.tensor([s for s, _ in rows], dtype=torch.int32,
                           device=run[0])
        want = torch.zeros(H, 10, R, dtype=F64)
        for i, (s, p) in enumerate(rows):
            lo = max(0, p + 1 - window) if window else 0
            kv = f64(lat[s][0])[lo:p + 1]
            sc = (f64(q_lat)[:, i] @ kv[:, :R].T +
                  f64(full)[i, :, D:] @ kv[:, R:].T) * scale
            want[:, i] = torch.softmax(sc, -1) @ kv[:, :R]
        for plain in (False, True):
            for ctx in (300, 5000):     # also more parts than there are keys
                got = ops.latent_decode(q_lat, full, cache, pos, seq, bt,
                                        window, scale, ctx, plain)
                close(got, want, run, f32=1e-5, bf16=1.2e-2)

    @pytest.mark.parametrize("window", [None, 1, 32, 33, 150])
    def test_prefill(self, run, H, D, rot, V, R, window):
        """Portions that start anywhere, behind rows of other sequences."""
        parts = [(3, 0), (140, 0), (40, 93), (9, 200), (129, 64)]
        rows = sum(n for n, _ in parts)
        base = parts[0][0]              # the first sequence is not ours
        seqs = [(n, prior, 0) for n, prior in parts]
        m, row_seq = meta(seqs, run)
        pos = torch.cat([torch.arange(prior, prior + n)
                         for n, prior in parts]).int()
        kv, lat, ctx, q = [], [], [(0, 0)], [rnd(3, H, D + rot)]
        want = torch.zeros(rows - base, H, V, dtype=F64)
        scale, at = 0.5, 0
        for s, (n, prior) in list(enumerate(parts))[1:]:
            first = max(0, prior + 1 - window) if window else 0
            t = prior + n - first
            k = rnd(t, D + rot, seed=60 + s)
            k = k / k.norm(dim=-1, keepdim=True) * 3
            kh = k[:, None, :D] * (1 + 0.1 * rnd(1, H, 1, seed=s))
            v = rnd(t, H, V, seed=70 + s)
            qq = stand_out(k, [prior + i - first for i in range(n)],
                           window, 2.0)[:, None].expand(n, H, D + rot)
            kv.append(torch.cat([kh.reshape(t, H * D),
                                 v.reshape(t, H * V)], 1))
            lat.append(torch.cat([rnd(t, R, seed=80 + s), k[:, D:]], 1))
            ctx.append((at, first))
            q.append(qq)
            at += t
        q = put(torch.cat(q), run)
        kvd, latd = put(torch.cat(kv), run), put(torch.cat(lat), run)
        for s, (n, prior) in list(enumerate(parts))[1:]:
            c0, first = ctx[s]
            r0 = sum(x for x, _ in parts[:s])
            t = prior + n - first
            k = f64(kvd)[c0:c0 + t, :H * D].view(t, H, D)
            v = f64(kvd)[c0:c0 + t, H * D:].view(t, H, V)
            qs = f64(q)[r0:r0 + n]
            p = prior + torch.arange(n)[:, None]
            j = first + torch.arange(t)[None, :]
            see = (j <= p) & (p - j < (window or prior + n))
            for h in range(H):
                sc = (qs[:, h, :D] @ k[:, h].T +
                      qs[:, h, D:] @ f64(latd)[c0:c0 + t, R:].T) * scale
                sc = sc.masked_fill(~see, -math.inf)
                want[r0 - base:r0 - base + n, h] = \
                    torch.softmax(sc, -1) @ v[:, h]
        want = want.reshape(rows - base, H * V)
        tiles = torch.tensor(
            [(s, r) for s, (n, _) in list(enumerate(parts))[1:]
             for r in range(0, n, layered.QUERY_TILE)], dtype=torch.int32,
            device=run[0])
        for plain in (False, True):
            out = torch.zeros(rows, H * V, dtype=run[1], device=run[0])
            ops.latent_prefill(q, kvd, latd, pos.to(run[0]), row_seq, base,
                               m, torch.tensor(ctx, dtype=torch.int32,
                                               device=run[0]),
                               tiles, rot, window, scale, out, plain)
            assert not out[:base].any()
            close(out[base:], want, run, f32=1e-5, bf16=1.2e-2)
