"""Runner for designs that list their layers (LayeredConfig).

One forward serves a mixed batch: single decoded tokens, short portions and
long portions of prompts side by side, in that order. Projections run over
all rows as one product each; mixers split the rows by what suits them:

  ChannelDelta     recurrent kernel for the first `n_step_seqs` sequences,
                   chunked kernels for the long portions after them
  LatentAttention  absorbed attention on the paged latents for the first
                   rows, expanded keys and values for the long portions

The residual stream is 32-bit; activations are `dtype` (bf16, or float32 for
exact runs). Mixers are independent of the design that lists them: a design
supplies a LayeredConfig and a `take(name)` function for its tensors.
"""
from dataclasses import dataclass
from typing import Callable, Dict, List, Optional, Tuple

import numpy as np
import torch

from ..ops import layered as ops
from .configs import (ChannelDeltaSpec, LatentAttentionSpec, LayeredConfig,
                      RotarySpec)
from . import rotary

# portions up to this many tokens run like decoded tokens
SHORT = 8
CHUNK = 64                  # tokens per chunk of the chunked recurrence
QUERY_TILE = 128            # query rows per workgroup of latent_prefill
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


def linear(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    return x @ w.t()


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
                               batch.seq_meta, origin, ctx["tiles"],
                               s.rot_dim, s.window, s.scale, out)
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
        self.mixers, self.norms, self.mlps, self.kv_layer = [], [], [], []
        self.windows = set()
        for i, layer in enumerate(config.layers):
            m = layer.mixer

            def mix(name, i=i):
                return take(f"l{i}.mix.{name}")
            if isinstance(m, ChannelDeltaSpec):
                self.mixers.append(ChannelDelta(m, mix, eps, dtype, device))
                self.kv_layer.append(i)
            else:
                if m.rot not in tables:
                    tables[m.rot] = rotary.table(m.rot, max_model_len, device)
                self.mixers.append(LatentAttention(m, mix, eps, dtype,
                                                   tables[m.rot]))
                self.kv_layer.append(i if m.kv_from is None else m.kv_from)
                self.windows.add(m.window)
            names = ("norm1", "norm1b") + (("norm2", "norm2b")
                                           if layer.ff else ())
            self.norms.append({x: take(f"l{i}.{x}").float() for x in names})
            self.mlps.append(None if not layer.ff else (
                torch.cat([take(f"l{i}.mlp.gate"),
                           take(f"l{i}.mlp.up")]).to(dtype),
                take(f"l{i}.mlp.down").to(dtype)))
        self.final_norm = take("final.norm").float()

    def weight_bytes(self) -> int:
        seen, total = set(), 0
        for obj in [self] + self.mixers:
            for t in vars(obj).values():
                if isinstance(t, torch.Tensor) and t.data_ptr() not in seen:
                    seen.add(t.data_ptr())
                    total += t.numel() * t.element_size()
        for pair in self.mlps:
            total += sum(t.numel() * t.element_size() for t in pair or ())
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

    def forward(self, batch: LayeredBatch, pool,
                embeddings_out: bool = False,
                layers_out: Optional[list] = None) -> torch.Tensor:
        """-> logits of `logit_rows` (or the normed stream of every row).
        layers_out collects copies of the stream after every layer."""
        c = self.cfg
        ctx = {}            # what layers of equal sizes share
        if batch.long:
            if self.windows:
                ctx["tiles"] = torch.tensor(
                    [(p.seq, r) for p in batch.long
                     for r in range(0, p.n, QUERY_TILE)],
                    dtype=torch.int32).to(self.device)
            for w in self.windows:
                ctx["keys", w] = self._context(batch, w, pool.block_size)
            for n in {m.per_group for m in self.mixers
                      if isinstance(m, ChannelDelta) and m.work}:
                ctx["chunks", n] = chunk_groups(batch.long, n, self.device)
        pre = [n["norm1"] for n in self.norms] + [self.final_norm]

        def norm(y, post, following):
            return ops.stream_norm(x, y, post, following, 1.0, c.rms_eps,
                                   self.dtype)
        x, h = ops.embed_norm(batch.input_ids, self.embed, c.embed_scale,
                              pre[0], 1.0, c.rms_eps)
        for i, mixer in enumerate(self.mixers):
            norms = self.norms[i]
            y = mixer(h, batch, pool.layers[self.kv_layer[i]], ctx)
            if self.mlps[i] is not None:
                h = norm(y, norms["norm1b"], norms["norm2"])
                gate_up, down = self.mlps[i]
                y = linear(ops.gelu_mul(linear(h, gate_up)), down)
                h = norm(y, norms["norm2b"], pre[i + 1])
            else:
                h = norm(y, norms["norm1b"], pre[i + 1])
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
