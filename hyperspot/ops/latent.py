"""Windowed latent attention: keys and values of all heads come from one row
[latent | rotated key part] per token in the pages.  A learned score without a
value may enter every head's softmax (`sink` [H] float), and a sigmoid of
`gate` [T, H] scale its output.

A GPU tensor runs the gfx950 kernels of csrc/attn_latent.hip, a CPU tensor the
PyTorch references.  Two ways to compute the same scores on the GPU:

  absorbed   the key expansion is applied to the query, W_uk^T q, and the head
             attends over the latents; the value expansion follows.  Decoded
             tokens and short portions: every cached row is read once for all
             heads.
  expanded   keys and values of the rows a portion sees are expanded per head
             first.  Longer portions: a third of the attention's work.
"""

from __future__ import annotations

import torch

from . import _native, torch_ref
from .hybrid import side_args


def rope_append(q, kv, w, meta, freqs, cache, heads: int, eps: float,
                gain: float = 1.0, side=None) -> None:
    """Rotate the last part of each head of q in place, cosine and sine times
    `gain`; append the normed latent (weight w) and rotated key part of kv, if
    the layer has its own.  `side`: an activation of the same rows."""
    rank = 0 if kv is None else w.numel()
    args = (q, kv, w, meta.positions, freqs, meta.slot_mapping, cache.kv,
            heads, rank, eps, gain)
    if q.is_cuda:
        _native().latent_rope_append(*args, *side_args(side))
        return
    torch_ref.latent_rope_append(*args)
    if side is not None:
        side.run_ref()


def attention(q, cache, meta, uk, uv, heads: int, window: int, scale: float,
              sink=None, gate=None, out=None) -> torch.Tensor:
    """[T, H*E] for q [T, H*(D+R)]; uk [rank, H*D], uv [H*E, rank].  `out` may
    be a column view of a wider buffer."""
    row_seq = meta.row_seq if meta.mode == "prefill" else None
    if out is None:
        out = torch.empty(q.shape[0], uv.shape[0], dtype=q.dtype,
                          device=q.device)
    if not q.is_cuda:
        return out.copy_(torch_ref.latent_attention(
            q, cache.kv, meta.block_tables, meta.positions, row_seq, uk, uv,
            heads, window, scale, sink, gate))
    span = None
    fits = _native().latent_fits(q, cache.kv, uk, uv, out, heads)
    if meta.mode == "prefill" and fits:
        span = meta.latent[window]
        if span.tiles.shape[0]:
            _expanded(out, q, cache, meta, span, uk, uv, heads, window, scale,
                      sink, gate)
        if span.rows is None:
            return out
    _absorbed(out, q, cache, meta, row_seq,
              None if span is None else span.rows, uk, uv, heads, window,
              scale, sink, gate, fits)
    return out


def _expanded(out, q, cache, meta, span, uk, uv, heads, window, scale, sink,
              gate):
    n, rank = _native(), uk.shape[0]
    lat = torch.empty(span.slots.numel(), cache.kv.shape[-1], dtype=q.dtype,
                      device=q.device)
    n.latent_gather(lat, cache.kv, span.slots)
    c = lat[:, :rank]
    n.latent_attn_prefill(
        out, q, c @ uk, lat, uv @ c.t(), meta.positions, meta.seq_start,
        span.start, span.first, span.tiles, heads, window, scale, sink, gate)


def _absorbed(out, q, cache, meta, row_seq, rows, uk, uv, heads, window,
              scale, sink, gate, fits):
    n, rank = _native(), uk.shape[0]
    R = q.shape[0] if rows is None else rows.numel()
    empty = lambda *s, dtype=q.dtype: torch.empty(*s, dtype=dtype,
                                                  device=q.device)
    qa = empty(R, heads, rank)
    n.latent_absorb(qa, q, uk, rows, heads)
    where = (cache.kv, meta.block_tables, meta.positions, rows, row_seq)
    if not fits:
        o = empty(R, heads, rank)
        n.latent_attn_general(o, qa, q, *where, window, scale, sink)
        n.latent_values(out, o, uv, rows, gate)
        return
    reach = min(window, meta.block_tables.shape[1] * cache.kv.shape[1])
    split = absorbed_split(R * -(-heads // 32), reach)
    if split == 1:
        o = empty(R, heads, rank)
        n.latent_attn_decode(o, qa, q, *where, 1, window, scale, sink)
        n.latent_values(out, o, uv, rows, gate)
    else:
        part = empty(R, heads, split, rank + 4, dtype=torch.float32)
        n.latent_attn_decode(part, qa, q, *where, split, window, scale, sink)
        n.latent_merge_values(out, part, uv, rows, R, heads, split, gate)


def absorbed_split(groups: int, reach: int) -> int:
    """How many workgroups share one row's window, each with at least 64
    tokens: one for every compute unit where few rows would give each many
    parts to combine, two otherwise.  Depends on shapes only, so a captured
    graph keeps it."""
    fill = 256 if groups < 128 else 512
    return max(1, min(16, fill // groups, reach // 64))
