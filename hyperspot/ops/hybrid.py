"""Ops of the hybrid designs (models.mixers), dispatched like the rest of the
op layer: a GPU tensor runs the gfx950 kernels of csrc/dyt.hip, csrc/rms.hip,
csrc/conv.hip, csrc/rope_norm.hip, csrc/attn_window.hip, csrc/attn_kept.hip,
csrc/attn_sigmoid.hip, csrc/recurrent.hip and csrc/recurrent_chunk.hip, a CPU
tensor the PyTorch references.

Dynamic-tanh parameters travel as tuples (w, b, alpha) of float tensors.
q, k, v, g are column views of one projection buffer [T, ...]; the kernels
take its row stride.
"""

from __future__ import annotations

from typing import NamedTuple, Optional

import torch

from . import _native, torch_ref


# ------------------------------------------------------ norms, feed-forward

def embed_dyt(table: torch.Tensor, ids: torch.Tensor, pre):
    """Token embedding into a float residual, and its first norm."""
    if table.is_cuda:
        T, W = ids.numel(), table.shape[1]
        res = torch.empty(T, W, dtype=torch.float32, device=table.device)
        out = torch.empty(T, W, dtype=table.dtype, device=table.device)
        _native().embed_dyt(out, res, table, ids, *pre)
        return out, res
    res = table[ids].float()
    return torch_ref.dyt(res, pre).to(table.dtype), res


def add_dyt(h: torch.Tensor, residual: torch.Tensor, post, pre):
    """residual += post(h) in place; returns pre(residual) in h's type."""
    if h.is_cuda:
        out = torch.empty_like(h)
        _native().add_dyt(out, residual, h, *post, *pre)
        return out
    residual += torch_ref.dyt(h, post)
    return torch_ref.dyt(residual, pre).to(h.dtype)


def embed_scaled(table: torch.Tensor, ids: torch.Tensor, scale: float):
    """(x, residual): the scaled embedding as float residual, and the same in
    the table's element type.  For a float table both are one tensor."""
    if not table.is_cuda:
        res = table[ids].float() * scale
        return res.to(table.dtype), res
    T, W = ids.numel(), table.shape[1]
    res = torch.empty(T, W, dtype=torch.float32, device=table.device)
    x = res if table.dtype == torch.float32 \
        else torch.empty(T, W, dtype=table.dtype, device=table.device)
    _native().embed_scaled(x, res, table, ids, scale)
    return x, res


def embed_residual(table: torch.Tensor, ids: torch.Tensor) -> torch.Tensor:
    """Token embedding as float residual only."""
    if not table.is_cuda:
        return table[ids].float()
    res = torch.empty(ids.numel(), table.shape[1], dtype=torch.float32,
                      device=table.device)
    _native().embed_scaled(None, res, table, ids, 1.0)
    return res


def rms_scale(x: torch.Tensor, w: torch.Tensor, eps: float, dtype):
    """RMS norm of float rows with a float weight, as `dtype`."""
    if not x.is_cuda:
        return torch_ref.rms_scale(x, w, eps).to(dtype)
    out = torch.empty(x.shape, dtype=dtype, device=x.device)
    _native().rms_scale(out, x, w, eps)
    return out


def add_rms(h: torch.Tensor, residual: torch.Tensor, w: torch.Tensor,
            eps: float, dtype) -> torch.Tensor:
    """residual += rms(h) * w in place; returns the residual as `dtype` (the
    residual itself for float)."""
    if not h.is_cuda:
        residual += torch_ref.rms_scale(h, w, eps)
        return residual.to(dtype)
    out = residual if dtype == torch.float32 \
        else torch.empty(h.shape, dtype=dtype, device=h.device)
    _native().add_rms(out, residual, h, w, eps)
    return out


class NextInput(NamedTuple):
    """How a sublayer's input is made of the residual: an RMS norm with
    weight `w` [W] and, if there is one, a causal convolution over time that
    is added to it.  `conv` [taps, W] float has the token's own tap last,
    `tail` [slots, taps - 1, W] the last inputs of every sequence."""

    w: torch.Tensor
    eps: float
    conv: Optional[torch.Tensor] = None
    tail: Optional[torch.Tensor] = None

    def row_args(self, meta):
        """Kernel arguments where a row is a sequence of its own."""
        if self.conv is None or meta.mode == "prefill":
            return None, None, None, None
        return self.conv, self.tail, meta.state_slots, meta.positions

    def finish(self, h, meta):
        """The convolution where the rows of a sequence meet each other."""
        if self.conv is None or meta.mode == "decode":
            return h
        return causal_conv(h, self.conv, self.tail, meta)


def next_input(residual: torch.Tensor, nxt: NextInput, meta,
               dtype) -> torch.Tensor:
    """The first sublayer's input."""
    if not residual.is_cuda:
        h = torch_ref.rms_scale(residual, nxt.w, nxt.eps).to(dtype)
        return _conv_ref(h, nxt, meta)
    h = torch.empty(residual.shape, dtype=dtype, device=residual.device)
    _native().add_rms_next(h, residual, None, None, nxt.w, nxt.eps,
                           *nxt.row_args(meta))
    return nxt.finish(h, meta)


def add_rms_next(y: torch.Tensor, residual: torch.Tensor, w: torch.Tensor,
                 nxt: NextInput, meta) -> torch.Tensor:
    """residual += rms(y) * w in place; returns the next sublayer's input in
    y's type."""
    if not y.is_cuda:
        residual += torch_ref.rms_scale(y, w, nxt.eps)
        h = torch_ref.rms_scale(residual, nxt.w, nxt.eps).to(y.dtype)
        return _conv_ref(h, nxt, meta)
    h = torch.empty_like(y)
    _native().add_rms_next(h, residual, y, w, nxt.w, nxt.eps,
                           *nxt.row_args(meta))
    return nxt.finish(h, meta)


def add_next(y: torch.Tensor, residual: torch.Tensor, nxt: NextInput,
             meta) -> torch.Tensor:
    """residual += y in place; returns the next sublayer's input in y's
    type."""
    if not y.is_cuda:
        residual += y.float()
        h = torch_ref.rms_scale(residual, nxt.w, nxt.eps).to(y.dtype)
        return _conv_ref(h, nxt, meta)
    h = torch.empty_like(y)
    _native().add_rms_next(h, residual, y, None, nxt.w, nxt.eps,
                           *nxt.row_args(meta))
    return nxt.finish(h, meta)


def _conv_ref(h, nxt: NextInput, meta):
    return h if nxt.conv is None \
        else causal_conv(h, nxt.conv, nxt.tail, meta)


def causal_conv(h: torch.Tensor, w: torch.Tensor, tail: torch.Tensor,
                meta) -> torch.Tensor:
    """h [T, W] plus its convolution over time within every sequence; the
    tails are renewed."""
    if not h.is_cuda:
        return torch_ref.causal_conv(
            h, w, tail, None if meta.mode == "decode" else meta.seq_start,
            meta.state_slots, meta.positions)
    out = torch.empty_like(h)
    _native().causal_conv(out, h, w, tail, meta.seq_start, meta.positions,
                          meta.state_slots, meta.tiles)
    return out


def rms_gate(o: torch.Tensor, g: torch.Tensor, w: torch.Tensor, eps: float,
             ss, total: int) -> torch.Tensor:
    """rms(o) * w * sigmoid(g) over the whole row of o [T, N] float.  `ss`
    [T] is the sum of squares of all `total` columns where o holds only some
    of them (None: o holds all)."""
    if not o.is_cuda:
        s = o.pow(2).sum(-1) if ss is None else ss
        y = o / (s / total + eps).sqrt()[:, None] * w
        return (y * torch.sigmoid(g.float())).to(g.dtype)
    y = torch.empty(o.shape, dtype=g.dtype, device=o.device)
    _native().rms_gate(y, o, g, w, ss, total, eps)
    return y


def row_squares(x: torch.Tensor) -> torch.Tensor:
    """Sum of squares of every row of x [T, N] float."""
    if not x.is_cuda:
        return x.pow(2).sum(-1)
    ss = torch.empty(x.shape[0], dtype=torch.float32, device=x.device)
    _native().row_squares(ss, x)
    return ss


def gelu_gate(z: torch.Tensor, table: torch.Tensor, ids: torch.Tensor,
              column: int) -> torch.Tensor:
    """gelu_tanh(z) * table[ids, column : column + n] for z [T, n]."""
    if not z.is_cuda:
        e = table[ids, column:column + z.shape[1]].float()
        return (torch.nn.functional.gelu(z.float(), approximate="tanh")
                * e).to(z.dtype)
    out = torch.empty_like(z)
    _native().gelu_gate(out, z, table, ids, column)
    return out


def gelu_mul(gate_up: torch.Tensor) -> torch.Tensor:
    """gelu_tanh(gate) * up for a merged [.., gate | up] projection."""
    if gate_up.is_cuda:
        out = torch.empty(*gate_up.shape[:-1], gate_up.shape[-1] // 2,
                          dtype=gate_up.dtype, device=gate_up.device)
        _native().gelu_mul(out, gate_up)
        return out
    return torch_ref.gelu_mul(gate_up)


def squared_relu(x: torch.Tensor) -> torch.Tensor:
    """relu(x)^2; in place on the GPU."""
    if x.is_cuda:
        _native().squared_relu(x)
        return x
    return x.float().clamp(min=0).square().to(x.dtype)


class SideRelu(NamedTuple):
    """out = relu(x)^2 for column views x, out [T, n] of two buffers, done by
    a kernel that has the same rows."""

    x: torch.Tensor
    out: torch.Tensor

    def run_ref(self) -> None:
        self.out.copy_(self.x.float().clamp(min=0).square())


def side_args(side: Optional[SideRelu]) -> tuple:
    return (None, None) if side is None else side


def clamped_glu(gate_up: torch.Tensor, limit: float) -> torch.Tensor:
    """g sigmoid(1.702 g) (u + 1) of a merged [gate | up] projection, with
    g = min(gate, limit) and u = up clamped to +-limit."""
    if not gate_up.is_cuda:
        return torch_ref.clamped_glu(gate_up, limit)
    out = torch.empty(*gate_up.shape[:-1], gate_up.shape[-1] // 2,
                      dtype=gate_up.dtype, device=gate_up.device)
    _native().clamped_glu(out, gate_up, limit)
    return out


# ---------------------------------------------------------------- attention

def rope_pairs_append(q, k, v, meta, freqs, cache, head_dim: int) -> None:
    """Interleaved rotary on q (in place) and k, append k and v to pages."""
    f = _native().rope_pairs_append if q.is_cuda \
        else torch_ref.rope_pairs_append
    f(q, k, v, meta.positions, freqs, meta.slot_mapping, cache.k, cache.v,
      head_dim)


def window_diff_attention(q, cache, meta, lam, window: int, scale: float,
                          diff: float, eps: float) -> torch.Tensor:
    """[T, H * E]; every row reads its keys from the pages (its own were
    appended just before)."""
    row_seq = meta.row_seq if meta.mode == "prefill" else None
    if not q.is_cuda:
        return torch_ref.window_diff_attention(
            q, cache.k, cache.v, meta.block_tables, meta.positions, row_seq,
            lam, window, scale, diff, eps)
    n, T = _native(), q.shape[0]
    G, E = cache.v.shape[1], cache.v.shape[2]
    H = q.shape[1] // cache.k.shape[3]
    out = torch.empty(T, H * E, dtype=q.dtype, device=q.device)
    if not n.window_attn_fits(q, cache.k, cache.v):
        n.window_attn_general(
            out, q, cache.k, cache.v, meta.block_tables, meta.positions,
            row_seq, lam, window, scale, diff, eps)
    elif meta.mode == "prefill":
        n.window_attn_prefill(
            out, q, cache.k, cache.v, meta.block_tables, meta.positions,
            meta.seq_start, meta.tiles, lam, window, scale, diff, eps)
    else:
        reach = min(window, meta.block_tables.shape[1] * cache.k.shape[2])
        split = decode_split(T * G * -(-(H // G) // 8), reach)
        partial = None if split == 1 else torch.empty(
            T * H * split * 2 * (E + 2), dtype=torch.float32,
            device=q.device)
        n.window_attn_decode(
            out, q, cache.k, cache.v, meta.block_tables, meta.positions, lam,
            partial, split, window, scale, diff, eps)
    return out


def rope_norm_append(q, k, v, meta, freqs, turn, cache, gain: float,
                     eps: Optional[float], side: Optional[SideRelu]) -> None:
    """Interleaved rotary on q (in place) and k, each head then divided by its
    root mean square (eps None: not); v turned over all its dimensions by the
    frequencies `turn` [E / 2] (empty: not); append k and v to pages."""
    if not q.is_cuda:
        torch_ref.rope_norm_append(q, k, v, meta.positions, freqs, turn,
                                   meta.slot_mapping, cache.k, cache.v, gain,
                                   eps)
        if side is not None:
            side.run_ref()
        return
    _native().rope_norm_append(q, k, v, meta.positions, freqs, turn,
                               meta.slot_mapping, cache.k, cache.v, gain, eps,
                               *side_args(side))


def window_attention(out, q, cache, meta, turn, sink, window: int, keep: int,
                     scale: float, bounded: bool = False) -> None:
    """out [T, H * E] (a column view): softmax attention over the last
    `window` positions and the first `keep`, `sink` [H] float in the
    denominators (None: nothing); outputs turned back by `turn`.  `bounded`:
    scores and sinks lie within +-40, so their exponentials need no running
    maximum."""
    row_seq = meta.row_seq if meta.mode == "prefill" else None
    if not q.is_cuda:
        torch_ref.window_attention(
            out, q, cache.k, cache.v, meta.block_tables, meta.positions,
            row_seq, turn, sink, window, keep, scale)
        return
    n, T = _native(), q.shape[0]
    G, E = cache.v.shape[1], cache.v.shape[2]
    H = q.shape[1] // cache.k.shape[3]
    where = (cache.k, cache.v, meta.block_tables, meta.positions)
    if not n.kept_attn_fits(out, q, cache.k, cache.v):
        n.kept_attn_general(out, q, *where, row_seq, turn, sink, window, keep,
                            scale)
    elif meta.mode == "prefill":
        n.kept_attn_prefill(out, q, *where, meta.seq_start, meta.tiles, turn,
                            sink, window, keep, scale, bounded)
    else:
        reach = min(window + keep,
                    meta.block_tables.shape[1] * cache.k.shape[2])
        split = decode_split(T * G * -(-(H // G) // 16), reach)
        partial = None if split == 1 else torch.empty(
            T * H * split * (E + 4), dtype=torch.float32, device=q.device)
        n.kept_attn_decode(out, q, *where, turn, sink, partial, split, window,
                           keep, scale, bounded)


def norm_append(q, k, v, qw, kw, meta, cache, eps: float) -> None:
    """RMS norm of every head of q (in place) and k, append k and v."""
    f = _native().norm_append if q.is_cuda else torch_ref.norm_append
    f(q, k, v, qw, kw, meta.slot_mapping, cache.k, cache.v, eps)


def sigmoid_attention(q, cache, meta, bias, chunk: int, scale: float,
                      cap: float) -> torch.Tensor:
    """[T, H * E]: the keys of a row's chunk up to itself, each weighing
    sigmoid(cap tanh(q.k scale / cap) + bias[h]); keys come from the pages."""
    row_seq = meta.row_seq if meta.mode == "prefill" else None
    if not q.is_cuda:
        return torch_ref.sigmoid_attention(
            q, cache.k, cache.v, meta.block_tables, meta.positions, row_seq,
            bias, chunk, scale, cap)
    n, T = _native(), q.shape[0]
    G, E = cache.v.shape[1], cache.v.shape[2]
    H = q.shape[1] // cache.k.shape[3]
    out = torch.empty(T, H * E, dtype=q.dtype, device=q.device)
    if not n.sigmoid_attn_fits(q, cache.k, cache.v):
        n.sigmoid_attn_general(
            out, q, cache.k, cache.v, meta.block_tables, meta.positions,
            row_seq, bias, chunk, scale, cap)
    elif meta.mode == "prefill":
        n.sigmoid_attn_prefill(
            out, q, cache.k, cache.v, meta.block_tables, meta.positions,
            meta.seq_start, meta.tiles, bias, chunk, scale, cap)
    else:
        reach = min(chunk, meta.block_tables.shape[1] * cache.k.shape[2])
        split = decode_split(T * G * -(-(H // G) // 16), reach)
        partial = None if split == 1 else torch.empty(
            T * H * split * E, dtype=torch.float32, device=q.device)
        n.sigmoid_attn_decode(
            out, q, cache.k, cache.v, meta.block_tables, meta.positions, bias,
            partial, split, chunk, scale, cap)
    return out


def decode_split(groups: int, reach: int) -> int:
    """How many workgroups share one row's window: enough to fill the chip
    when the batch alone does not, each with at least 128 tokens.  Depends on
    shapes only, so a captured graph keeps it."""
    return max(1, min(16, 512 // groups, reach // 128))


# ---------------------------------------------------------------- recurrent

def gla_mix(q, k, v, g, a1h, a2, a2b, w, state, meta, tau: float,
            eps: float) -> torch.Tensor:
    """Gated linear attention of one layer up to its output projection."""
    _, H, D, E = state.S.shape
    T, qscale = q.shape[0], D ** -0.5
    decode = meta.mode == "decode"
    if not q.is_cuda:
        o = torch_ref.gla_scan(
            q, k, v, torch_ref.gla_log_decay(a1h, a2, a2b, tau), state,
            None if decode else meta.seq_start, meta.state_slots,
            meta.positions, qscale)
        return torch_ref.recurrent_out(o, g, w, "silu", eps, q.dtype)
    n = _native()
    y = torch.empty(T, H * E, dtype=q.dtype, device=q.device)
    if decode:
        n.gla_step(y, state.S, q, k, v, g, a1h, a2, a2b, w, meta.positions,
                   meta.state_slots, qscale, tau, eps)
        return y
    if n.chunk_fits(state.S, q, k, v, g, a2.shape[1]):
        b = torch.empty(T, H * D, dtype=torch.float32, device=q.device)
        n.gla_chunk_gates(b, a1h, a2, a2b, meta.seq_start, meta.tiles, tau)
        U = torch.empty(meta.tiles.shape[0], H, E, D, dtype=torch.float32,
                        device=q.device)
        n.recurrent_chunk(y, U, None, None, state.S, None, None, q, k, v, g,
                          b, None, w, meta.seq_start, meta.positions,
                          meta.state_slots, meta.tiles, meta.tile_start,
                          qscale, eps)
        return y
    decay = torch.empty(T, H * D, dtype=torch.float32, device=q.device)
    n.gla_decay(decay, a1h, a2, a2b, tau)
    o = torch.empty(T, H, E, dtype=torch.float32, device=q.device)
    n.recurrent_scan(o, state.S, None, None, None, q, k, v, decay,
                     meta.seq_start, meta.positions, meta.state_slots, qscale)
    n.recurrent_out(y, o, g, w, H, False, eps)
    return y


def mlstm_mix(q, k, v, g, raw, ib, fb, w, state, meta, cap: float,
              eps: float) -> torch.Tensor:
    """Matrix LSTM of one layer up to its output projection; `raw` [T, 2H]
    float holds the input and forget gate projections."""
    _, H, D, E = state.S.shape
    T, qscale = q.shape[0], D ** -0.5
    decode = meta.mode == "decode"
    if not q.is_cuda:
        i, f = torch_ref.mlstm_log_gates(raw, ib, fb, cap)
        o = torch_ref.mlstm_scan(
            q, k, v, i, f, state, None if decode else meta.seq_start,
            meta.state_slots, meta.positions, qscale)
        return torch_ref.recurrent_out(o, g, w, "sigmoid", eps, q.dtype)
    n = _native()
    y = torch.empty(T, H * E, dtype=q.dtype, device=q.device)
    if decode:
        n.mlstm_step(y, state.S, state.n, state.m, q, k, v, g, raw, ib, fb, w,
                     meta.positions, meta.state_slots, qscale, cap, eps)
        return y
    gates = torch.empty_like(raw)
    if n.chunk_fits(state.S, q, k, v, g, 0):
        f32 = lambda *s: torch.empty(meta.tiles.shape[0], H, *s,
                                     dtype=torch.float32, device=q.device)
        info, U, nU, m_in = f32(2), f32(E, D), f32(D), f32()
        n.mlstm_chunk_gates(gates, info, raw, ib, fb, meta.seq_start,
                            meta.tiles, cap)
        n.recurrent_chunk(y, U, nU, m_in, state.S, state.n, state.m, q, k, v,
                          g, gates, info, w, meta.seq_start, meta.positions,
                          meta.state_slots, meta.tiles, meta.tile_start,
                          qscale, eps)
        return y
    n.mlstm_gates(gates, raw, ib, fb, cap)
    o = torch.empty(T, H, E, dtype=torch.float32, device=q.device)
    nm = torch.empty(meta.state_slots.numel(), H, D + 1, dtype=torch.float32,
                     device=q.device)
    n.recurrent_scan(o, state.S, state.n, state.m, nm, q, k, v, gates,
                     meta.seq_start, meta.positions, meta.state_slots, qscale)
    n.recurrent_out(y, o, g, w, H, True, eps)
    return y


def lightning_mix(q, k, v, decay, state, meta) -> torch.Tensor:
    """Lightning attention of one layer before its norm, [T, H*E] float; SiLU
    is applied to q, k and v on the way in."""
    _, H, D, E = state.S.shape
    T = q.shape[0]
    decode = meta.mode == "decode"
    if not q.is_cuda:
        return torch_ref.lightning_scan(
            q, k, v, decay, state, None if decode else meta.seq_start,
            meta.state_slots, meta.positions).view(T, H * E)
    n = _native()
    o = torch.empty(T, H * E, dtype=torch.float32, device=q.device)
    if decode:
        n.lightning_step(o, state.S, q, k, v, decay, meta.positions,
                         meta.state_slots)
    elif n.chunk_fits(state.S, q, k, v, v, 0):
        U = torch.empty(meta.tiles.shape[0], H, E, D, dtype=torch.float32,
                        device=q.device)
        n.lightning_chunk(o, U, state.S, q, k, v, decay, meta.seq_start,
                          meta.positions, meta.state_slots, meta.tiles,
                          meta.tile_start)
    else:
        n.lightning_scan(o, state.S, q, k, v, decay, meta.seq_start,
                         meta.positions, meta.state_slots)
    return o


def gate_projection(h: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """h @ w^T with a float result: gate logits are not rounded to bf16."""
    if h.dtype == torch.float32:
        return h @ w.t()
    if h.is_cuda:
        return torch.mm(h, w.t(), out_dtype=torch.float32)
    return h.float() @ w.float().t()
