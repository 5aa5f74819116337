"""Ops of grouped attention, experts and the looped stream one by one against
the plain oracle: the CPU versions everywhere, the HIP kernels in both
precisions on a GPU."""
import pytest
import torch

import sezazen_oracle as oracle
from llm_d_inference_scheduler_amd.ops import layered as ops
from test_layered_ops import F64, GPU, RUNS, close, f64, meta, put, rnd

F32 = ("", torch.float32)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("width", [38, 64, 1000, 4096, 9000])
class TestStream:
    def test_embedding_with_positions(self, run, width):
        table, pos = put(rnd(11, width), run), rnd(9, width, seed=4)
        ids = torch.tensor([3, 0, 10, 3], device=run[0])
        at = torch.tensor([0, 8, 3, 7], dtype=torch.int32, device=run[0])
        wn = rnd(width, seed=3)
        want = f64(table)[ids.cpu()] * 2.5 + pos.double()[at.cpu().long()]
        x, h = ops.embed_norm(ids, table, 2.5, wn.to(run[0]), 0.0, 1e-3,
                              pos.to(run[0]), at)
        assert x.dtype == torch.float32
        assert (f64(x) - want).abs().max() < 1e-5
        close(h, oracle.rms_norm(want, wn.double(), 1e-3), run)
        x, h = ops.embed_norm(ids, table, 2.5, None, 0.0, 1e-3,
                              pos.to(run[0]), at)      # no norm: a copy
        assert torch.equal(h, x.to(run[1]))

    @pytest.mark.parametrize("n", [0, 1, 3])
    @pytest.mark.parametrize("has_y", [True, False])
    def test_sum(self, run, width, n, has_y):
        x, y = rnd(5, width), put(rnd(5, width, seed=1), run)
        rows = put(rnd(5 * n, width, seed=2), run) if n else None
        wn = rnd(width, seed=3)
        xd = x.clone().to(run[0])
        h = ops.stream_norm(xd, y if has_y else None, None, wn.to(run[0]),
                            0.0, 1e-3, run[1], rows)
        want = x.double()
        if has_y:
            want = want + f64(y)
        if n:
            want = want + f64(rows).view(5, n, width).sum(1)
        assert (f64(xd) - want).abs().max() < 3e-6      # stays 32-bit
        close(h, oracle.rms_norm(want, wn.double(), 1e-3), run)
        h = ops.stream_norm(xd, None, None, None, 0.0, 1e-3, run[1])
        assert torch.equal(h, xd.to(run[1]))

    def test_loop_entry(self, run, width):
        a, b, v = rnd(5, width), rnd(5, width, seed=1), rnd(width, seed=2)
        wn = rnd(width, seed=3)
        x = torch.full((5, width), float("nan"), device=run[0])
        h = ops.loop_norm(x, a.to(run[0]), b.to(run[0]), v.to(run[0]),
                          wn.to(run[0]), 0.0, 1e-3, run[1])
        want = a.double() + b.double() + v.double()
        assert (f64(x) - want).abs().max() < 3e-6
        close(h, oracle.rms_norm(want, wn.double(), 1e-3), run)


@pytest.mark.parametrize("run", RUNS)
class TestActivations:
    @pytest.mark.parametrize("size", [22, 64])
    def test_silu_gate(self, run, size):
        gu = put(rnd(7, 2 * size, scale=4), run)
        gu[0, 0], gu[0, 1] = 90.0, -90.0
        close(ops.gated_act(gu, "silu"),
              oracle.silu(f64(gu)[:, :size]) * f64(gu)[:, size:], run)

    @pytest.mark.parametrize("size", [22, 64])
    def test_relu_squared(self, run, size):
        x = put(rnd(7, size, scale=4), run)
        close(ops.activate(x, "relu_squared"), oracle.relu_squared(f64(x)),
              run)

    def test_linear32(self, run):
        x, w = put(rnd(33, 72), run), put(rnd(40, 72, seed=1), run)
        y = ops.linear32(x, w)
        assert y.dtype == torch.float32
        close(y, f64(x) @ f64(w).T, F32, f32=2e-6)


# ---- grouped attention ------------------------------------------------------
BS = 16


def paged(run, G, D, V, ctxs, seed=0):
    """-> cache with scattered pages, block tables, [(k, v)] in 64-bit. Pages
    that no sequence owns hold values that would show."""
    blocks = sum(-(-c // BS) for c in ctxs) + 3
    g = torch.Generator().manual_seed(seed)
    order = torch.randperm(blocks, generator=g).tolist()
    cache = torch.full((blocks, G, BS, D + V), 50.0)
    tables = torch.zeros(len(ctxs), max(-(-c // BS) for c in ctxs) + 1,
                         dtype=torch.int32)
    kv = []
    for s, c in enumerate(ctxs):
        k, v = rnd(c, G, D, seed=seed + s), rnd(c, G, V, seed=seed + 50 + s)
        k, v = k.to(run[1]), v.to(run[1])
        kv.append([k.double(), v.double()])
        for t in range(c):
            if t % BS == 0:
                tables[s, t // BS] = order.pop()
            cache[tables[s, t // BS], :, t % BS] = torch.cat(
                [k[t], v[t]], -1).float()
    return put(cache, run), tables.to(run[0]), kv


def expected(q, k, v, pos, scale, sink):
    """q [H, D] at position pos; k [T, G, D], v [T, G, V] -> [H V]."""
    H, G = q.shape[0], k.shape[1]
    out = []
    for h in range(H):
        g = h // (H // G)
        s = (k[:pos + 1, g] @ q[h] * scale)[None]
        see = torch.ones_like(s, dtype=torch.bool)
        p = oracle.sink_softmax(s, see) if sink is not None \
            else torch.softmax(s, -1)
        out.append(p @ v[:pos + 1, g])
    return torch.cat(out, -1)[0]


# H, G, D, V: vector and odd sizes, one to many heads per group
HEADS = [(4, 2, 16, 24), (6, 1, 24, 8), (3, 3, 7, 5), (20, 1, 40, 72),
         (8, 2, 128, 128), (33, 1, 64, 16), (4, 2, 192, 256), (2, 1, 12, 40)]


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("H,G,D,V", HEADS)
class TestGroupedAttention:
    def test_store(self, run, H, G, D, V):
        proj = put(rnd(7, H * D + G * (D + V) + 8), run)
        cache = put(torch.full((4, G, BS, D + V), 9.0), run)
        before = cache.clone()
        slots = torch.tensor([3, 60, 15, 16, 17, 0, 63], device=run[0])
        ops.store_heads(proj, H * D, slots, cache, D)
        for i, s in enumerate(slots.tolist()):
            got = cache[s // BS, :, s % BS]
            split = H * D + G * D
            assert torch.equal(got[:, :D].flatten(),
                               proj[i, H * D:split])
            assert torch.equal(got[:, D:].flatten(),
                               proj[i, split:split + G * V])
            before[s // BS, :, s % BS] = got
        assert torch.equal(cache, before)

    @pytest.mark.parametrize("plain", [False, True])
    @pytest.mark.parametrize("sink", [0.0, None, 1.5])
    def test_decode(self, run, H, G, D, V, plain, sink):
        if sink == 1.5:
            def want_row(q, k, v, pos):     # exp(1.5) in the sum
                k2 = torch.cat([torch.zeros_like(k[:1]), k])
                v2 = torch.cat([torch.zeros_like(v[:1]), v])
                out = []
                for h in range(H):
                    g = h // (H // G)
                    s = k2[:pos + 2, g] @ q[h] * scale
                    s[0] = 1.5
                    out.append(torch.softmax(s, -1) @ v2[:pos + 2, g])
                return torch.cat(out)
        else:
            def want_row(q, k, v, pos):
                return expected(q, k, v, pos, scale, sink)
        ctxs = [1, 2, 15, 16, 17, 63, 64, 65, 129, 300, 700]
        if plain:
            ctxs = [1, 17, 300]
        scale = 1.2 * D ** -0.5
        cache, tables, kv = paged(run, G, D, V, ctxs)
        n = len(ctxs)
        proj = put(rnd(n + 2, H * D + G * (D + V), seed=3), run)
        pos = torch.tensor([c - 1 for c in ctxs] + [0, 0], dtype=torch.int32)
        seq = torch.arange(n + 2, dtype=torch.int32)
        out = put(torch.full((n + 2, H * V), 7.0), run)
        ops.grouped_decode(proj, cache, pos.to(run[0]), seq.to(run[0]),
                           tables, n, H, D, scale, sink, max(ctxs), out,
                           plain=plain)
        q = f64(proj)[:, :H * D].view(n + 2, H, D)
        want = torch.stack([want_row(q[i], *kv[i], ctxs[i] - 1)
                            for i in range(n)])
        close(out[:n], want, run, f32=5e-6)
        assert (out[n:] == 7).all()

    @pytest.mark.parametrize("plain", [False, True])
    @pytest.mark.parametrize("sink", [0.0, None])
    def test_prefill(self, run, H, G, D, V, plain, sink):
        """Portions with and without earlier tokens, around tile sizes."""
        portions = [(0, 64), (17, 70), (200, 9), (63, 130)]
        if plain:
            portions = [(0, 20), (17, 9)]
        scale = 1.2 * D ** -0.5
        cache, tables, kv = paged(run, G, D, V, [a + n for a, n in portions])
        base = 3        # decoded rows in front: not touched
        seqs, pos = [], [0] * base
        for i, (prior, n) in enumerate(portions):
            seqs.append((n, prior, 0))
            pos += range(prior, prior + n)
        m, rows = meta(seqs, run)
        m[:, 0] += base
        rows = torch.cat([torch.zeros_like(rows[:base]), rows])
        T = base + sum(n for _, n in portions)
        per = max(1, 128 * G // H)
        tiles = torch.tensor([(i, r) for i, (_, n) in enumerate(portions)
                              for r in range(0, n, per)], dtype=torch.int32)
        proj = put(rnd(T, H * D + G * (D + V), seed=3), run)
        out = put(torch.full((T, H * V), 7.0), run)
        ops.grouped_prefill(
            proj, cache, torch.tensor(pos, dtype=torch.int32).to(run[0]),
            rows, tables, base, m, tiles.to(run[0]), H, D, scale, sink, out,
            plain=plain)
        q = f64(proj)[:, :H * D].view(T, H, D)
        want, row = [], base
        for (prior, n), (k, v) in zip(portions, kv):
            for t in range(n):
                want.append(expected(q[row], k, v, prior + t, scale, sink))
                row += 1
        close(out[base:], torch.stack(want), run, f32=5e-6)
        assert (out[:base] == 7).all()

    def test_one_key_stands_out(self, run, H, G, D, V):
        """A key far back, at page and tile borders, and the token's own: the
        output is that key's value, in decoding and in a portion. The key
        after the query would win as well if it were seen."""
        ctx = 520
        for at in (0, 15, 16, 63, 64, 128, 447, 448, 511, 518):
            cache, tables, kv = paged(run, G, D, V, [ctx], seed=at)
            k, v = kv[0]
            strong = 40.0 * torch.ones(D, dtype=F64) / D ** 0.5
            for t, x in ((at, strong), (519, 1.5 * strong)):
                blk = tables[0, t // BS]
                cache[blk, :, t % BS, :D] = x.to(cache)
            q = torch.ones(1, H, D) / D ** 0.5
            proj = torch.cat([q.flatten(1), torch.zeros(1, G * (D + V))], 1)
            want = torch.cat([v[at, h // (H // G)] for h in range(H)])
            for n in (1, 200):      # one row; the last of a portion
                T, prior = n, 519 - n
                p = put(proj.expand(T, -1), run)
                pos = torch.arange(prior, prior + n, dtype=torch.int32,
                                   device=run[0])
                seq = torch.zeros(T, dtype=torch.int32, device=run[0])
                out = put(torch.zeros(T, H * V), run)
                if n == 1:
                    ops.grouped_decode(p, cache, pos, seq, tables, 1, H, D,
                                       1.0, 0.0, 519, out)
                else:
                    m, _ = meta([(n, prior, 0)], run)
                    per = max(1, 128 * G // H)
                    tiles = torch.tensor([(0, r) for r in range(0, n, per)],
                                         dtype=torch.int32, device=run[0])
                    ops.grouped_prefill(p, cache, pos, seq, tables, 0, m,
                                        tiles, H, D, 1.0, 0.0, out)
                close(out[-1], want, run, f32=1e-5)


# ---- experts ----------------------------------------------------------------
@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("T,K,E,top", [
    (1, 38, 5, 2), (17, 64, 3, 3), (40, 200, 16, 1), (33, 64, 33, 8),
    (5, 72, 100, 4), (16, 128, 256, 7), (9, 64, 300, 2)])
class TestRoute:
    def test_choice_and_scores(self, run, T, K, E, top):
        h, w = put(rnd(T, K), run), put(rnd(E, K, seed=1, scale=K ** -0.5),
                                        run)
        ids, wt = ops.route(h, w, top)
        assert ids.dtype == torch.int32 and wt.dtype == torch.float32
        want_ids, want = oracle.route(f64(h), f64(w), top)
        # sums differ in order only: scores agree, and so do clear choices
        close(wt, want, F32, f32=1e-5)
        s = oracle.sigmoid(f64(h) @ f64(w).T)
        ids = ids.cpu().long()
        assert all(len(set(r)) == top for r in ids.tolist())
        assert (torch.gather(s, 1, ids) - want).abs().max() < 1e-5

    def test_ties_go_to_the_lower_expert(self, run, T, K, E, top):
        h, w = put(rnd(T, K), run), put(torch.zeros(E, K), run)
        ids, wt = ops.route(h, w, top)
        assert ids.tolist() == [list(range(top))] * T
        assert (wt == 0.5).all()


SHAPES = [(38, 11, 5), (64, 24, 7), (64, 64, 4), (192, 320, 6), (128, 200, 3)]


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("K,F,E", SHAPES)
class TestExperts:
    """Pairs per expert from one to hundreds: each form of the kernels."""

    def weights(self, run, K, F, E):
        return (put(rnd(E, F, K, seed=2, scale=K ** -0.5), run),
                put(rnd(E, K, F, seed=3, scale=F ** -0.5), run))

    def want(self, h, ids, wt, up, down):
        h, up, down, wt = f64(h), f64(up), f64(down), f64(wt)
        out = torch.zeros(ids.numel(), h.shape[1], dtype=F64)
        for p, e in enumerate(ids.flatten().tolist()):
            t = p // ids.shape[1]
            out[p] = oracle.expert(wt.flatten()[p] * h[t][None], up[e],
                                   down[e])[0]
        return out

    @pytest.mark.parametrize("T,top", [(1, 1), (3, 2), (50, 3), (130, 2),
                                       (400, 2)])
    def test_products(self, run, K, F, E, T, top):
        g = torch.Generator().manual_seed(T)
        up, down = self.weights(run, K, F, E)
        h = put(rnd(T, K), run)
        wt = (torch.rand(T, top, generator=g) * 0.9 + 0.05)
        ids = torch.stack([torch.randperm(E, generator=g)[:top]
                           for _ in range(T)]).int()
        out = ops.experts(h, ids.to(run[0]), wt.to(run[0]), up, down,
                          "relu_squared")
        want = self.want(h, ids, wt, up, down)
        close(out, want, run, f32=1e-5, bf16=2e-2)
        # the weight belongs to the input: on the output it would show
        bare = self.want(h, ids, torch.ones_like(wt), up, down)
        other = bare * wt.flatten()[:, None]
        assert (other - want).abs().max() > 0.1 * want.abs().max()

    def test_one_expert_takes_all(self, run, K, F, E):
        T = 150
        up, down = self.weights(run, K, F, E)
        h, wt = put(rnd(T, K), run), torch.full((T, 1), 0.7)
        ids = torch.full((T, 1), E - 1, dtype=torch.int32)
        ids[77] = 0
        out = ops.experts(h, ids.to(run[0]), wt.to(run[0]), up, down,
                          "relu_squared")
        close(out, self.want(h, ids, wt, up, down), run, f32=1e-5, bf16=2e-2)

    def test_rows_do_not_depend_on_the_batch(self, run, K, F, E):
        """A token alone and in a crowd."""
        up, down = self.weights(run, K, F, E)
        h = put(rnd(300, K), run)
        wt = torch.full((300, 2), 0.5, device=run[0])
        ids = torch.tensor([[1, 2], [0, 1], [2, 0]], dtype=torch.int32,
                           device=run[0]).repeat(100, 1)
        many = ops.experts(h, ids, wt, up, down, "relu_squared")
        for t in (0, 7, 299):
            one = ops.experts(h[t:t + 1].contiguous(),
                              ids[t:t + 1].contiguous(), wt[:1], up, down,
                              "relu_squared")
            close(one, f64(many[2 * t:2 * t + 2]), run, f32=1e-5, bf16=2e-2)


@GPU
def test_forms_agree_at_a_large_size():
    """The tiled products against the plain kernel."""
    dev, E, K, F, T, top = "cuda:0", 9, 512, 448, 1500, 3
    g = torch.Generator(device=dev).manual_seed(0)

    def normal(*shape, std=1.0):
        return torch.empty(shape, device=dev).normal_(
            0, std, generator=g).bfloat16()
    up, down = normal(E, F, K, std=K ** -0.5), normal(E, K, F, std=F ** -0.5)
    h = normal(T, K)
    ids, wt = ops.route(h, normal(E, K, std=K ** -0.5), top)
    a = ops.experts(h, ids, wt, up, down, "relu_squared")
    b = ops.experts(h, ids, wt, up, down, "relu_squared", plain=True)
    close(a, f64(b), ("", torch.bfloat16), bf16=1e-2)
