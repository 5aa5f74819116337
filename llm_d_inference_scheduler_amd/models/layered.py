"""Runner for designs that list their layers (LayeredConfig).

One forward serves a mixed batch: single decoded tokens, short portions and
long portions of prompts side by side, in that order. Projections run over
all rows as one product each; mixers split the rows by what suits them:

  ChannelDelta     recurrent kernel for the first `n_step_seqs` sequences,
                   chunked kernels for the long portions after them
  LatentAttention  absorbed attention on the paged latents for the first
                   rows, expanded keys and values for the long portions
  GroupedAttention both straight on the pages: parts of the context for the
                   first rows, query tiles for the long portions

The order of the forward is config.runs: a looped stretch of layers runs
several times, every pass with caches of its own.

The residual stream is 32-bit; activations are `dtype` (bf16, or float32 for
exact runs). Mixers are independent of the design that lists them: a design
supplies a LayeredConfig and a `take(name)` function for its tensors.
"""
from dataclasses import dataclass
from typing import Callable, Dict, List, Optional, Tuple

import numpy as np
import torch

from ..ops import layered as ops
from ..ops.layered import linear
from .configs import (ChannelDeltaSpec, GroupedAttentionSpec,
                      LatentAttentionSpec, LayeredConfig, RotarySpec)
from . import feed_forward, rotary

# portions up to this many tokens run like decoded tokens
SHORT = 8
CHUNK = 64                  # tokens per chunk of the chunked recurrence
QUERY_TILE = 128            # query rows per workgroup of the prefill kernels
WORK_BYTES = 160 << 20      # its workspace: stays in the last-level cache


@dataclass
class Portion:
    """A portion of a prompt inside a batch (host view)."""
    seq: int                # sequence index in the batch
    row0: int
    n: int
    prior: int              # tokens of the sequence before the portion
    table: List[int]        # its blocks
    slot: int               # its recurrent-state slot


@dataclass
class ChunkGroup:
    """Chunks of long portions that run with one workspace."""
    chunks: torch.Tensor        # [n, 2] int32: first row, tokens
    walk: torch.Tensor          # [s, 4] int32: first row, tokens, state slot,
    chunks_host: torch.Tensor   # first chunk | 1 << 30 (state starts at zero)
    walk_host: torch.Tensor


def chunk_groups(long: List[Portion], per_group: int,
                 device: torch.device) -> List[ChunkGroup]:
    """Cut long portions into chunks, at most `per_group` a group. A group
    takes a stretch of every portion in turn (they run side by side); the
    next group goes on from the stored states."""
    total = sum(-(-p.n // CHUNK) for p in long)
    per_group = -(-total // -(-total // per_group))     # groups of like size
    groups = []
    at = [0] * len(long)
    while any(a < p.n for a, p in zip(at, long)):
        left = sum(a < p.n for a, p in zip(at, long))
        chunks, walk = [], []
        for i, p in enumerate(long):
            if at[i] == p.n or len(chunks) == per_group:
                continue
            share = max(1, (per_group - len(chunks)) // left)
            left -= 1
            n = min(p.n - at[i], share * CHUNK)
            row = p.row0 + at[i]
            fresh = p.prior + at[i] == 0
            walk.append((row, n, p.slot, len(chunks) | fresh << 30))
            chunks.extend((row + a, min(CHUNK, n - a))
                          for a in range(0, n, CHUNK))
            at[i] += n
        c = torch.tensor(chunks, dtype=torch.int32)
        w = torch.tensor(walk, dtype=torch.int32)
        groups.append(ChunkGroup(c.to(device), w.to(device), c, w))
    return groups


@dataclass
class LayeredBatch:
    """Rows of `n_step_seqs` short sequences first, then long portions."""
    input_ids: torch.Tensor         # [T] int64
    positions: torch.Tensor         # [T] int32
    slot_mapping: torch.Tensor      # [T] int64, cache slot of every row
    row_seq: torch.Tensor           # [T] int32
    seq_meta: torch.Tensor          # [S, 4] int32: row0, rows, prior, slot
    block_tables: torch.Tensor      # [S, max_blocks] int32
    n_step_seqs: int
    n_step_rows: int
    multi_row: bool                 # some sequence has more than one row
    max_ctx: int                    # longest context among the step rows
    long: List[Portion]
    logit_rows: Optional[torch.Tensor] = None   # None: every row


class ChannelDelta:
    """Gated delta rule with one decay per head and key channel."""

    def __init__(self, spec: ChannelDeltaSpec, take: Callable, eps: float,
                 dtype: torch.dtype, device: torch.device):
        self.spec, self.eps = spec, eps

        def act(name):
            return take(name).to(dtype)
        self.work = ops.delta_chunk_work(spec.dim, spec.vdim, device)
        self.per_group = max(1, WORK_BYTES // max(
            1, self.work * spec.heads * 4))
        self.w_in = torch.cat([act(n) for n in ("q", "k", "v", "b", "a1",
                                                "g1")])
        self.beta_col = spec.conv_channels
        self.a_col = self.beta_col + spec.heads
        self.g_col = self.a_col + spec.decay_rank
        self.w_a2, self.w_g2, self.w_o = act("a2"), act("g2"), act("o")
        self.taps = torch.cat([take(n + ".conv").float()
                               for n in ("q", "k", "v")]).t().contiguous()
        self.neg_a = -torch.exp(take("A_log").float())
        self.dt_bias = take("dt_bias").float()
        self.norm = take("norm").float()

    def __call__(self, h: torch.Tensor, batch: LayeredBatch, cache,
                 ctx) -> torch.Tensor:
        s = self.spec
        conv_state, state = cache
        proj = linear(h, self.w_in)
        decay = linear(proj[:, self.a_col:self.g_col], self.w_a2)
        gate = linear(proj[:, self.g_col:], self.w_g2)
        q, k, v = ops.delta_prep(
            proj, self.taps, conv_state, batch.row_seq, batch.seq_meta,
            batch.multi_row, s.kv_heads, s.heads, s.dim, s.vdim,
            s.dim ** -0.5, s.unit_eps)
        T = h.shape[0]
        out = torch.empty((T, s.heads * s.vdim), dtype=h.dtype,
                          device=h.device)
        chunked = batch.long and self.work
        ops.delta_step(q, k, v, proj, self.beta_col, decay, self.dt_bias,
                       self.neg_a, gate, self.norm, state, batch.seq_meta,
                       batch.n_step_seqs if chunked
                       else batch.seq_meta.shape[0], out, self.eps)
        if chunked:
            o = torch.empty((T, s.heads * s.vdim), dtype=torch.float32,
                            device=h.device)
            groups = ctx["chunks", self.per_group]
            ws = torch.empty(self.work * s.heads * max(
                len(g.chunks_host) for g in groups), dtype=torch.float32,
                device=h.device)
            for g in groups:
                ops.delta_chunk(q, k, v, proj, self.beta_col, decay,
                                self.dt_bias, self.neg_a, state, g, ws, o)
            ops.delta_gate(o, gate, self.norm, out, batch.n_step_rows,
                           self.eps)
        return linear(out, self.w_o)


class LatentAttention:
    """Attention over cached latents (its own layer's or an earlier one's)."""

    def __init__(self, spec: LatentAttentionSpec, take: Callable, eps: float,
                 dtype: torch.dtype, cos_sin: torch.Tensor):
        self.spec, self.eps, self.cos_sin = spec, eps, cos_sin

        def act(name):
            return take(name).to(dtype)
        own = spec.kv_from is None
        self.w_in = torch.cat([act("dq"), act("dkv")]) if own else act("dq")
        self.q_norm = take("dq.norm").float()
        self.kv_norm = take("dkv.norm").float() if own else None
        self.w_uq, self.w_o = act("uq"), act("o")
        uk, uv = act("uk"), act("uv")
        self.w_ukv = torch.cat([uk, uv])         # expands keys and values
        # absorbing products, one matrix per head
        self.w_uk = self.w_ukv[:uk.shape[0]].view(spec.heads, spec.dim,
                                                  spec.kv_rank)
        self.w_uv = uv.view(spec.heads, spec.vdim, spec.kv_rank).transpose(
            1, 2).contiguous()

    def __call__(self, h: torch.Tensor, batch: LayeredBatch, cache,
                 ctx) -> torch.Tensor:
        s, n = self.spec, batch.n_step_rows
        T = h.shape[0]
        proj = linear(h, self.w_in)
        cq = ops.latent_prep(proj, self.q_norm, self.kv_norm, self.cos_sin,
                             batch.positions, batch.slot_mapping,
                             cache if s.kv_from is None else None, self.eps)
        q = linear(cq, self.w_uq).view(T, s.heads, s.dim + s.rot_dim)
        q_plain = ops.rope_part(q, self.cos_sin, batch.positions, n)
        out = torch.empty((T, s.heads * s.vdim), dtype=h.dtype,
                          device=h.device)
        if n:
            q_lat = torch.bmm(q_plain, self.w_uk)
            o_lat = ops.latent_decode(q_lat, q, cache, batch.positions,
                                      batch.row_seq, batch.block_tables,
                                      s.window, s.scale, batch.max_ctx)
            ops.heads_to_rows(torch.bmm(o_lat, self.w_uv), out)
        if n < T:
            slots, origin = ctx["keys", s.window]
            lat = ops.gather_rows(cache, slots)
            kv = linear(lat[:, :s.kv_rank], self.w_ukv)
            ops.latent_prefill(q, kv, lat, batch.positions, batch.row_seq, n,
                               batch.seq_meta, origin,
                               ctx["tiles", QUERY_TILE],
                               s.rot_dim, s.window, s.scale, out)
        return linear(out, self.w_o)


class GroupedAttention:
    """Attention of grouped heads over paged keys and values."""

    def __init__(self, spec: GroupedAttentionSpec, take: Callable,
                 dtype: torch.dtype):
        self.spec = spec
        self.w_in = torch.cat([take(n) for n in "qkv"]).to(dtype)
        self.w_o = take("o").to(dtype)

    @property
    def tile_rows(self) -> int:
        """Queries of a portion per tile: the heads of a group share it."""
        return max(1, QUERY_TILE * self.spec.kv_heads // self.spec.heads)

    def __call__(self, h: torch.Tensor, batch: LayeredBatch, cache,
                 ctx) -> torch.Tensor:
        s, n = self.spec, batch.n_step_rows
        T = h.shape[0]
        proj = linear(h, self.w_in)
        ops.store_heads(proj, s.heads * s.dim, batch.slot_mapping, cache,
                        s.dim)
        out = torch.empty((T, s.heads * s.vdim), dtype=h.dtype,
                          device=h.device)
        if n:
            ops.grouped_decode(proj, cache, batch.positions, batch.row_seq,
                               batch.block_tables, n, s.heads, s.dim,
                               s.scale, s.sink, batch.max_ctx, out)
        if n < T:
            ops.grouped_prefill(proj, cache, batch.positions, batch.row_seq,
                                batch.block_tables, n, batch.seq_meta,
                                ctx["tiles", self.tile_rows], s.heads, s.dim,
                                s.scale, s.sink, out)
        return linear(out, self.w_o)


class LayeredRunner:
    mixed_batches = True        # decode rows and portions share one forward

    def __init__(self, config: LayeredConfig, take: Callable,
                 device: torch.device, dtype: torch.dtype,
                 max_model_len: int = 8192):
        self.cfg, self.device, self.dtype = config, device, dtype
        eps = config.rms_eps
        tables: Dict[RotarySpec, torch.Tensor] = {}
        self.embed = take("embed").to(dtype)
        self.lm_head = self.embed
        self.positions = take("pos").float() if config.learned_positions \
            else None
        self.runs = config.runs
        self.loop_x = self.loop_x0 = self.loop_step = None
        if config.loop:
            w = take("loop.in").to(dtype)
            self.loop_x = w[:, :config.hidden_size].contiguous()
            self.loop_x0 = w[:, config.hidden_size:].contiguous()
            self.loop_step = take("loop.step").float()
        self.mixers, self.norms, self.mlps = [], [], []
        self.windows = set()
        for i, layer in enumerate(config.layers):
            m = layer.mixer

            def mix(name, i=i):
                return take(f"l{i}.mix.{name}")

            def mlp(name, i=i):
                return take(f"l{i}.mlp.{name}")
            if isinstance(m, ChannelDeltaSpec):
                self.mixers.append(ChannelDelta(m, mix, eps, dtype, device))
            elif isinstance(m, GroupedAttentionSpec):
                self.mixers.append(GroupedAttention(m, mix, dtype))
            else:
                if m.rot not in tables:
                    tables[m.rot] = rotary.table(m.rot, max_model_len, device)
                self.mixers.append(LatentAttention(m, mix, eps, dtype,
                                                   tables[m.rot]))
                self.windows.add(m.window)
            names = ("norm1",) + ("norm2",) * bool(layer.ff)
            if config.post_norms:
                names += tuple(n + "b" for n in names)
            self.norms.append({x: take(f"l{i}.{x}").float() for x in names})
            self.mlps.append(layer.ff and feed_forward.build(layer.ff, mlp,
                                                             dtype))
        self.final_norm = take("final.norm").float()
        # query tiles the prefill kernels take, by queries per tile
        self.tile_rows = {m.tile_rows for m in self.mixers
                          if isinstance(m, GroupedAttention)}
        if self.windows:
            self.tile_rows.add(QUERY_TILE)

    def weight_bytes(self) -> int:
        seen, total = set(), 0
        for obj in [self] + self.mixers + [m for m in self.mlps if m]:
            for t in vars(obj).values():
                if isinstance(t, torch.Tensor) and t.data_ptr() not in seen:
                    seen.add(t.data_ptr())
                    total += t.numel() * t.element_size()
        return total

    # ------------------------------------------------------------------
    def _context(self, batch: LayeredBatch, window: Optional[int],
                 block_size: int) -> Tuple[torch.Tensor, torch.Tensor]:
        """Cache slots of every key the long portions may see, and each
        sequence's (first context row, its position)."""
        origin = np.zeros((batch.seq_meta.shape[0], 2), dtype=np.int32)
        slots, row = [], 0
        for p in batch.long:
            first = max(0, p.prior + 1 - window) if window else 0
            t = np.arange(first, p.prior + p.n, dtype=np.int64)
            table = np.asarray(p.table, dtype=np.int64)
            slots.append(table[t // block_size] * block_size + t % block_size)
            origin[p.seq] = row, first
            row += len(t)
        return (torch.from_numpy(np.concatenate(slots)).to(self.device),
                torch.from_numpy(origin).to(self.device))

    def _shared_inputs(self, batch: LayeredBatch, block_size: int) -> dict:
        """What layers of equal sizes share about the long portions."""
        ctx = {}
        if not batch.long:
            return ctx
        for n in self.tile_rows:
            ctx["tiles", n] = torch.tensor(
                [(p.seq, r) for p in batch.long for r in range(0, p.n, n)],
                dtype=torch.int32).to(self.device)
        for w in self.windows:
            ctx["keys", w] = self._context(batch, w, block_size)
        for n in {m.per_group for m in self.mixers
                  if isinstance(m, ChannelDelta) and m.work}:
            ctx["chunks", n] = chunk_groups(batch.long, n, self.device)
        return ctx

    def forward(self, batch: LayeredBatch, pool,
                embeddings_out: bool = False,
                layers_out: Optional[list] = None) -> torch.Tensor:
        """-> logits of `logit_rows` (or the normed stream of every row).
        layers_out collects copies of the stream after every layer run."""
        c, runs = self.cfg, self.runs
        ctx = self._shared_inputs(batch, pool.block_size)
        # the norm ahead of every run; a run that enters a loop pass takes
        # the stream itself (None)
        pre = [None if r.enters is not None else self.norms[r.layer]["norm1"]
               for r in runs] + [self.final_norm]

        def update(y, rows, post, following):
            return ops.stream_norm(x, y, post, following, c.norm_offset,
                                   c.rms_eps, self.dtype, rows)
        x, h = ops.embed_norm(batch.input_ids, self.embed, c.embed_scale,
                              pre[0], c.norm_offset, c.rms_eps,
                              self.positions, batch.positions)
        if c.loop:      # the embedding output's share is the same every pass
            x0 = ops.linear32(h if pre[0] is None else x.to(self.dtype),
                              self.loop_x0)
        for i, run in enumerate(runs):
            norms, mlp = self.norms[run.layer], self.mlps[run.layer]
            if run.enters is not None:
                h = ops.loop_norm(x, ops.linear32(h, self.loop_x), x0,
                                  self.loop_step[run.enters], norms["norm1"],
                                  c.norm_offset, c.rms_eps, self.dtype)
            y = self.mixers[run.layer](h, batch, pool.layers[run.cache], ctx)
            h = update(y, None, norms.get("norm1b"),
                       norms["norm2"] if mlp else pre[i + 1])
            if mlp:
                h = update(*mlp(h), norms.get("norm2b"), pre[i + 1])
            if layers_out is not None:
                layers_out.append(x.clone())
        if embeddings_out:
            return h
        if batch.logit_rows is not None:
            h = h[batch.logit_rows]
        return self.project(h)

    def project(self, h: torch.Tensor) -> torch.Tensor:
        """Normed stream -> logits."""
        return linear(h, self.lm_head)
