"""Dispatch of the layer-listed designs' ops: `_hip_layered` on GPU tensors
(required there, no eager fallback), `ref_layered` on CPU tensors."""
import torch

from . import ref_layered as ref

try:
    from .. import _hip_layered as _ext
except ImportError:  # extension not built
    _ext = None


def hip_layered():
    """The raw extension module. Fail-loud."""
    if _ext is None:
        raise RuntimeError(
            "_hip_layered extension is not built; run "
            "`python setup.py build_ext --inplace`")
    return _ext


def _impl(t: torch.Tensor):
    return hip_layered() if t.is_cuda else ref


# activation codes of the kernels
ACTS = {"gelu_tanh": 0, "silu": 1, "relu_squared": 2}


def linear(x, w):
    return x @ w.t()


def linear32(x, w):
    """x @ w' with a 32-bit result."""
    if x.is_cuda and x.dtype != torch.float32:
        return torch.mm(x, w.t(), out_dtype=torch.float32)
    return x.float() @ w.float().t()


def embed_norm(ids, table, scale, wn, offset, eps, pos=None, positions=None):
    """-> (stream x = table[ids] * scale (+ pos[positions]) in 32-bit, its
    norm; without wn x itself in the table's type)."""
    return _impl(table).embed_norm(ids, table, scale, wn, offset, eps, pos,
                                   positions)


def stream_norm(x, y, wb, wn, offset, eps, dtype, rows=None):
    """In place: x += rms_norm(y) * (wb + offset), without wb x += y, without
    y nothing; with rows [T * n, width] also each token's n rows.
    -> rms_norm(x) * (wn + offset) as dtype; without wn x as dtype."""
    return _impl(x).stream_norm(x, y, wb, wn, offset, eps,
                                dtype == torch.float32, rows)


def loop_norm(x, a, b, v, wn, offset, eps, dtype):
    """In place: x = a + b + v (a vector); -> its norm as in stream_norm."""
    return _impl(x).loop_norm(x, a, b, v, wn, offset, eps,
                              dtype == torch.float32)


def gated_act(gate_up, act):
    """act(gate) * up on packed rows."""
    return _impl(gate_up).gated_act(gate_up, ACTS[act])


def activate(x, act):
    return _impl(x).activate(x, ACTS[act])


def route(h, w, top):
    """-> (experts [T, top] int32 with the largest scores sigmoid(h w'),
    largest first, and these scores), scores in 32-bit."""
    return _impl(h).route(h, w, top)


def experts(h, ids, weights, up, down, act, plain=False):
    """down[e] act(up[e] (weight h)) of every token's experts e, rows
    [T * top, width] in the order of ids."""
    return _impl(h).experts(h, ids, weights, up, down, ACTS[act], plain)


def delta_prep(proj, taps, conv_state, row_seq, seq_meta, multi_row, kv_heads,
               heads, dim, vdim, q_scale, unit_eps):
    """Short convolutions, silu and unit norms -> 32-bit q, k, v; the
    convolution inputs of every sequence move on in conv_state."""
    return _impl(proj).delta_prep(proj, taps, conv_state, row_seq, seq_meta,
                                  multi_row, kv_heads, heads, dim, vdim,
                                  q_scale, unit_eps)


def delta_step(q, k, v, proj, beta_col, decay, dt_bias, neg_a, gate, norm_w,
               state, seq_meta, n_seqs, out, eps):
    """Token-by-token recurrence of the first n_seqs sequences."""
    _impl(q).delta_step(q, k, v, proj, beta_col, decay, dt_bias, neg_a, gate,
                        norm_w, state, seq_meta, n_seqs, out, eps)


def delta_chunk_work(dim, vdim, device):
    """Floats of workspace per (chunk, head); 0 without a chunked form (then
    delta_step takes every sequence)."""
    return hip_layered().delta_chunk_work(dim, vdim) \
        if device.type == "cuda" else 0


def delta_chunk(q, k, v, proj, beta_col, decay, dt_bias, neg_a, state, group,
                ws, out):
    """Chunked recurrence of the sequences of one ChunkGroup -> 32-bit out."""
    hip_layered().delta_chunk(q, k, v, proj, beta_col, decay, dt_bias, neg_a,
                              state, group.chunks, group.walk,
                              group.chunks_host, group.walk_host, ws, out)


def delta_gate(o, gate, norm_w, out, base, eps):
    """Gated output norm of the rows from `base` on."""
    hip_layered().delta_gate(o, gate, norm_w, out, base, eps)


def latent_prep(proj, wq, wkv, cos_sin, positions, slots, cache, eps):
    """Norm of the query latent; latent and rotated key part -> cache."""
    return _impl(proj).latent_prep(proj, wq, wkv, cos_sin, positions, slots,
                                   cache, eps)


def rope_part(q, cos_sin, positions, n_abs):
    """Rotates the last dims of every head in place; -> the unrotated part
    of the first n_abs rows, by head."""
    return _impl(q).rope_part(q, cos_sin, positions, n_abs)


def heads_to_rows(src, dst):
    _impl(src).heads_to_rows(src, dst)


def gather_rows(cache, slots):
    return _impl(cache).gather_rows(cache, slots)


def latent_decode(q_lat, q, cache, positions, row_seq, block_tables, window,
                  scale, max_ctx, plain=False):
    """Absorbed attention of single rows over the paged latents."""
    return _impl(q).latent_decode(q_lat, q, cache, positions, row_seq,
                                  block_tables, window or 0, scale, max_ctx,
                                  plain)


def latent_prefill(q, kv, lat, positions, row_seq, base, seq_meta, ctx, tiles,
                   rot, window, scale, out, plain=False):
    """Attention of the rows from `base` on over expanded keys and values."""
    _impl(q).latent_prefill(q, kv, lat, positions, row_seq, base, seq_meta,
                            ctx, tiles, rot, window or 0, scale, out, plain)


def store_heads(proj, col, slots, cache, dim):
    """Keys of all heads, then values of all heads, from column `col` on ->
    the cache pages [blocks, heads, tokens, key | value]."""
    _impl(proj).store_heads(proj, col, slots, cache, dim)


def grouped_decode(proj, cache, positions, row_seq, block_tables, n, heads,
                   dim, scale, sink, max_ctx, out, plain=False):
    """Attention of the first n rows (queries lead the rows of proj) over the
    paged keys and values; sink: score of a key without a value, or None."""
    _impl(proj).grouped_decode(proj, cache, positions, row_seq, block_tables,
                               n, heads, dim, scale, sink, max_ctx, out,
                               plain)


def grouped_prefill(proj, cache, positions, row_seq, block_tables, base,
                    seq_meta, tiles, heads, dim, scale, sink, out,
                    plain=False):
    """The same for the rows from `base` on; tiles [n, 2] = (sequence, first
    row of its portion)."""
    _impl(proj).grouped_prefill(proj, cache, positions, row_seq,
                                block_tables, base, seq_meta, tiles, heads,
                                dim, scale, sink, out, plain)
