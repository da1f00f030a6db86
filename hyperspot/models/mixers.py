"""Layer parts of the hybrid designs: norms, mixers, feed-forwards, token
inputs.

A mixer takes the normed input, the step's metadata and its layer's cache and
returns the branch output before the post-norm.  Its sizes and constants come
from its spec in engine.layer_spec, so a design is a list of specs plus the
order in which its blocks apply norms.

Projections of one input are merged into one GEMM; the merged output is read
through strided column views.  `tensors(prefix)` lists the checkpoint tensors
of a part: (name, full shape, setter).
"""

from __future__ import annotations

import torch
from torch import nn

from hyperspot.engine.layer_spec import (DiffAttention, Experts, GatedLinear,
                                         LatentAttention, Lightning,
                                         MatrixLSTM, SigmoidAttention,
                                         SquaredRelu, WindowAttention)
from hyperspot.engine.rotary import (frequencies, gain, head_order,
                                     pair_order)
from hyperspot.ops import experts, hybrid, latent
from hyperspot.parallel import (MergedColumnParallelLinear,
                                MergedRowParallelLinear, RowParallelLinear)
from hyperspot.parallel.layers import _init_weight
from hyperspot.parallel.state import (get_ep_size, get_tp_rank, get_tp_size,
                                      tensor_model_parallel_all_reduce)


def _param(t: torch.Tensor) -> nn.Parameter:
    return nn.Parameter(t, requires_grad=False)


def _random(shape, tag: int, std: float = 0.02) -> torch.Tensor:
    n = 1
    for s in shape:
        n *= s
    return (_init_weight(1, n, torch.float32, tag) * (std / 0.02)).view(shape)


def _rows(param: nn.Parameter, tp: int, r: int, full: int) -> nn.Parameter:
    """Mark a parameter as sharded over dimension 0 for checkpoint save."""
    if tp > 1:
        n = full // tp
        param._tp_shard_dim = 0
        param._tp_slices = [(r * n, n, 0)]
        param._tp_full_shape = (full,) + tuple(param.shape[1:])
    return param


def _put(param: nn.Parameter, tp: int = 1, r: int = 0):
    """Setter that keeps rank r's block of dimension 0."""
    def put(full: torch.Tensor) -> None:
        n = full.shape[0] // tp if full.dim() else 0
        part = full[r * n:(r + 1) * n] if tp > 1 else full
        param.data.copy_(part.reshape(param.shape))
    return put


def _shard(param: nn.Parameter, dim: int, slices: list, full_shape: tuple):
    """Mark a parameter as sharded over `dim` for checkpoint save."""
    if get_tp_size() > 1:
        param._tp_shard_dim, param._tp_slices = dim, slices
        param._tp_full_shape = full_shape
    return param


def _part(layer, i: int):
    return lambda full: layer.load_part(i, full)


class DynamicTanh(nn.Module):
    """Statistics-free norm tanh(alpha x) w + b, parameters in float."""

    def __init__(self, width: int):
        super().__init__()
        self.w = _param(torch.ones(width))
        self.b = _param(torch.zeros(width))
        self.alpha = _param(torch.full((1,), 0.5))

    @property
    def args(self) -> tuple:
        return self.w, self.b, self.alpha

    def tensors(self, name: str):
        n = self.w.numel()
        yield name, (n,), _put(self.w)
        yield name + ".b", (n,), _put(self.b)
        yield name + ".alpha", (), _put(self.alpha)


class RmsScale(nn.Module):
    """RMS norm with a float weight; `stored` is what a checkpoint's weight
    is short of the factor (1 for weights stored around zero)."""

    def __init__(self, width: int, stored: float = 0.0):
        super().__init__()
        self.w = _param(torch.ones(width))
        self.stored = stored

    def tensors(self, name: str):
        yield name, tuple(self.w.shape), \
            lambda t: self.w.data.copy_(t.float() + self.stored)


class GatedGelu(nn.Module):
    """down(gelu_tanh(gate x) * up x)."""

    def __init__(self, width: int, ff: int, dtype, tag: int):
        super().__init__()
        self.gate_up = MergedColumnParallelLinear(width, [ff, ff], dtype,
                                                  seed_tag=tag)
        self.down = RowParallelLinear(ff, width, dtype, seed_tag=tag + 2)
        self.width, self.ff = width, ff

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return self.down(hybrid.gelu_mul(self.gate_up(x)))

    def tensors(self, p: str):
        yield p + "gate", (self.ff, self.width), _part(self.gate_up, 0)
        yield p + "up", (self.ff, self.width), _part(self.gate_up, 1)
        yield p + "down", (self.width, self.ff), self.down.load_full_weight


class SquaredReluMLP(nn.Module):
    """down(relu(up x)^2)."""

    def __init__(self, spec: SquaredRelu, width: int, dtype, tag: int):
        super().__init__()
        self.up = MergedColumnParallelLinear(width, [spec.ff], dtype,
                                             seed_tag=tag)
        self.down = RowParallelLinear(spec.ff, width, dtype, seed_tag=tag + 1)
        self.width, self.ff = width, spec.ff

    def add_next(self, x, residual, norm: RmsScale, nxt, meta):
        """residual += norm(self(x)); the next sublayer's input."""
        y = self.down(hybrid.squared_relu(self.up(x)))
        return hybrid.add_rms_next(y, residual, norm.w, nxt, meta)

    def tensors(self, p: str):
        yield p + "up", (self.ff, self.width), _part(self.up, 0)
        yield p + "down", (self.width, self.ff), self.down.load_full_weight


class ExpertMixture(nn.Module):
    """Gated experts chosen per token, and an optional shared one.

    Under tensor parallelism every expert's inner size is divided over the
    ranks, so all ranks run all experts and the sum is one all-reduce."""

    def __init__(self, spec: Experts, width: int, dtype, tag: int):
        super().__init__()
        if get_ep_size() > 1:
            raise ValueError("this design's experts are divided over the "
                             "tensor-parallel group; ep_size must be 1")
        self.spec, self.width = spec, width
        m, tp, r = spec, get_tp_size(), get_tp_rank()

        def pair(count, ff, tag):
            """([count, gate | up, width], [count, width, ff]) of this rank"""
            assert ff % tp == 0, (ff, tp)
            n = ff // tp
            a = _init_weight(count * 2 * ff, width, dtype, tag) \
                .view(count, 2, ff, width)[:, :, r * n:(r + 1) * n]
            b = _init_weight(count * width, ff, dtype, tag + 1) \
                .view(count, width, ff)[:, :, r * n:(r + 1) * n]
            up = _param(a.reshape(count, 2 * n, width).contiguous())
            down = _param(b.contiguous())
            return (_shard(up, 1, [(r * n, n, 0), (ff + r * n, n, n)],
                           (count, 2 * ff, width)),
                    _shard(down, 2, [(r * n, n, 0)], (count, width, ff)))

        self.up, self.down = pair(m.experts, m.ff, tag)
        self.shared_up = self.shared_down = None
        if m.shared is not None:
            self.shared_up, self.shared_down = pair(1, m.shared, tag + 2)
        # router rows, then the shared expert's gate: one product
        self.routes = m.experts + m.identity
        self.router = _param(_init_weight(
            self.routes + (m.shared is not None), width, dtype, tag + 4))
        self.correction = _param(torch.zeros(self.routes)) if m.over_all \
            else None

    @property
    def args(self) -> tuple:
        return (self.router, self.up, self.down, self.shared_up,
                self.shared_down, self.spec.top)

    @property
    def rules(self) -> experts.Rules:
        return experts.Rules(self.correction, self.spec.identity,
                             self.spec.limit, get_tp_rank() == 0)

    def add_normed(self, x, residual, norm: RmsScale, eps: float):
        """residual += norm(mixture of x); the residual in x's type."""
        if get_tp_size() == 1:
            return experts.mixture_add_rms(x, *self.args, residual, norm.w,
                                           eps, self.rules)
        y = tensor_model_parallel_all_reduce(
            experts.mixture(x, *self.args, self.rules))
        return hybrid.add_rms(y, residual, norm.w, eps, x.dtype)

    def add_next(self, x, residual, norm: RmsScale, nxt, meta):
        """residual += norm(mixture of x); the next sublayer's input."""
        if get_tp_size() == 1:
            return experts.mixture_add_next(x, *self.args, self.rules,
                                            residual, norm.w, nxt, meta)
        y = tensor_model_parallel_all_reduce(
            experts.mixture(x, *self.args, self.rules))
        return hybrid.add_rms_next(y, residual, norm.w, nxt, meta)

    def tensors(self, p: str):
        m, w = self.spec, self.width
        tp, r = get_tp_size(), get_tp_rank()

        def expert(p, up, down, ff):
            n = ff // tp
            yield p + "gate", (ff, w), \
                lambda t: up[:n].copy_(t[r * n:(r + 1) * n])
            yield p + "up", (ff, w), \
                lambda t: up[n:].copy_(t[r * n:(r + 1) * n])
            yield p + "down", (w, ff), \
                lambda t: down.copy_(t[:, r * n:(r + 1) * n])

        for i in range(m.experts):
            yield from expert(f"{p}e{i}.", self.up.data[i],
                              self.down.data[i], m.ff)
        n = self.routes
        yield p + "router", (n, w), self.router.data[:n].copy_
        if self.correction is not None:
            yield p + "correction", (n,), self.correction.data.copy_
        if m.shared is not None:
            yield from expert(p + "shared.", self.shared_up.data[0],
                              self.shared_down.data[0], m.shared)
            yield p + "shared.sg", (1, w), self.router.data[n:].copy_


class InputConv(nn.Module):
    """Causal convolution over time on each channel of a sublayer's input,
    added to it; weights in float, kept [taps, width]."""

    def __init__(self, width: int, taps: int, tag: int):
        super().__init__()
        self.w = _param(_random((taps, width), tag, 0.1))

    def tensors(self, name: str):
        yield name, tuple(self.w.t().shape), \
            lambda t: self.w.data.copy_(t.t())


class TokenSide(nn.Module):
    """A token's own input to one layer: the residual gates the token's entry
    of a table, the product is projected, normed and added."""

    def __init__(self, width: int, dim: int, column: int, dtype, tag: int):
        super().__init__()
        self.width, self.dim, self.column = width, dim, column
        whole = lambda i, o, t: MergedColumnParallelLinear(
            i, [o], dtype, seed_tag=t, replicated=(0,))
        self.gate = whole(width, dim, tag)
        self.proj = whole(dim, width, tag + 1)
        self.norm = RmsScale(width)

    def add(self, x, residual, table, ids, eps: float):
        """residual += this layer's input; the residual in x's type."""
        g = hybrid.gelu_gate(self.gate(x), table, ids, self.column)
        return hybrid.add_rms(self.proj(g), residual, self.norm.w, eps,
                              x.dtype)

    def tensors(self, p: str):
        yield p + "gate", (self.dim, self.width), _part(self.gate, 0)
        yield p + "proj", (self.width, self.dim), _part(self.proj, 0)
        yield from self.norm.tensors(p + "norm")


class WindowDiffAttention(nn.Module):
    def __init__(self, spec: DiffAttention, width: int, eps: float, dtype,
                 tag: int):
        super().__init__()
        self.spec, self.width, self.eps = spec, width, eps
        m = spec
        self.qkv = MergedColumnParallelLinear(
            width, [m.heads * 2 * m.dim, m.kv_heads * 2 * m.dim,
                    m.kv_heads * m.vdim], dtype, seed_tag=tag)
        self.o_proj = RowParallelLinear(m.heads * m.vdim, width, dtype,
                                        seed_tag=tag + 3)
        # rows lq1, lk1, lq2, lk2
        self.lam = _param(_random((4, m.dim), tag + 4, 0.1))
        i = torch.arange(0, m.rot_dims, 2, dtype=torch.float64)
        self.register_buffer(
            "freqs", m.rot_base ** (-i / m.rot_dims) if m.rot_dims else i,
            persistent=False)

    def forward(self, x, meta, cache) -> torch.Tensor:
        m = self.spec
        q, k, v = self.qkv.split(self.qkv(x))
        hybrid.rope_pairs_append(q, k, v, meta, self.freqs, cache, m.dim)
        o = hybrid.window_diff_attention(q, cache, meta, self.lam, m.window,
                                         m.scale, m.diff, self.eps)
        return self.o_proj(o)

    def tensors(self, p: str):
        m, w = self.spec, self.width
        yield p + "q", (m.heads * 2 * m.dim, w), _part(self.qkv, 0)
        yield p + "k", (m.kv_heads * 2 * m.dim, w), _part(self.qkv, 1)
        yield p + "v", (m.kv_heads * m.vdim, w), _part(self.qkv, 2)
        yield p + "o", (w, m.heads * m.vdim), self.o_proj.load_full_weight
        for i, n in enumerate(("lq1", "lk1", "lq2", "lk2")):
            yield p + n, (m.dim,), lambda t, i=i: self.lam.data[i].copy_(t)


class GatedLinearAttention(nn.Module):
    def __init__(self, spec: GatedLinear, width: int, eps: float, dtype,
                 tag: int):
        super().__init__()
        self.spec, self.width, self.eps = spec, width, eps
        m = spec
        d, e = m.heads * m.dim, m.heads * m.vdim
        # q | k | v | g | first half of the decay projection (kept whole)
        self.proj = MergedColumnParallelLinear(
            width, [d, d, e, e, m.rank], dtype, seed_tag=tag,
            replicated=(4,))
        self.o_proj = RowParallelLinear(e, width, dtype, seed_tag=tag + 5)
        tp, r = get_tp_size(), get_tp_rank()
        n = d // tp
        self.a2 = _rows(_param(_init_weight(d, m.rank, dtype, tag + 6)
                               [r * n:(r + 1) * n].contiguous()), tp, r, d)
        self.a2_b = _rows(_param(torch.zeros(n)), tp, r, d)
        self.norm = _param(torch.ones(m.vdim))

    def forward(self, x, meta, state) -> torch.Tensor:
        q, k, v, g, a1h = self.proj.split(self.proj(x))
        return self.o_proj(hybrid.gla_mix(
            q, k, v, g, a1h, self.a2, self.a2_b, self.norm, state, meta,
            self.spec.tau, self.eps))

    def tensors(self, p: str):
        m, w = self.spec, self.width
        d, e = m.heads * m.dim, m.heads * m.vdim
        tp, r = get_tp_size(), get_tp_rank()
        for i, (n, rows) in enumerate((("q", d), ("k", d), ("v", e),
                                       ("g", e), ("a1", m.rank))):
            yield p + n, (rows, w), _part(self.proj, i)
        yield p + "o", (w, e), self.o_proj.load_full_weight
        yield p + "a2", (d, m.rank), _put(self.a2, tp, r)
        yield p + "a2.b", (d,), _put(self.a2_b, tp, r)
        yield p + "norm", (m.vdim,), _put(self.norm)


class MatrixMemoryLSTM(nn.Module):
    def __init__(self, spec: MatrixLSTM, width: int, eps: float, dtype,
                 tag: int):
        super().__init__()
        self.spec, self.width, self.eps = spec, width, eps
        m = spec
        d, e = m.heads * m.dim, m.heads * m.vdim
        self.proj = MergedColumnParallelLinear(width, [d, d, e, e], dtype,
                                               seed_tag=tag)
        # input | forget gate logits, a GEMM of their own with float output
        self.gates = MergedColumnParallelLinear(
            width, [m.heads, m.heads], dtype, seed_tag=tag + 4)
        self.o_proj = RowParallelLinear(e, width, dtype, seed_tag=tag + 6)
        tp, r = get_tp_size(), get_tp_rank()
        hs, es = m.heads // tp, e // tp
        self.i_b = _rows(_param(torch.zeros(hs)), tp, r, m.heads)
        self.f_b = _rows(_param(torch.zeros(hs)), tp, r, m.heads)
        self.norm = _rows(_param(torch.ones(es)), tp, r, e)

    def forward(self, x, meta, state) -> torch.Tensor:
        q, k, v, g = self.proj.split(self.proj(x))
        raw = hybrid.gate_projection(x, self.gates.weight)
        return self.o_proj(hybrid.mlstm_mix(
            q, k, v, g, raw, self.i_b, self.f_b, self.norm, state, meta,
            self.spec.gate_cap, self.eps))

    def tensors(self, p: str):
        m, w = self.spec, self.width
        d, e = m.heads * m.dim, m.heads * m.vdim
        tp, r = get_tp_size(), get_tp_rank()
        for i, (n, rows) in enumerate((("q", d), ("k", d), ("v", e),
                                       ("g", e))):
            yield p + n, (rows, w), _part(self.proj, i)
        yield p + "o", (w, e), self.o_proj.load_full_weight
        yield p + "norm", (e,), _put(self.norm, tp, r)
        for i, (n, b) in enumerate((("i", self.i_b), ("f", self.f_b))):
            yield p + n, (m.heads, w), _part(self.gates, i)
            yield p + n + ".b", (m.heads,), _put(b, tp, r)


class ChunkedSigmoidAttention(nn.Module):
    def __init__(self, spec: SigmoidAttention, width: int, eps: float, dtype,
                 tag: int):
        super().__init__()
        self.spec, self.width, self.eps = spec, width, eps
        m, tp, r = spec, get_tp_size(), get_tp_rank()
        self.qkv = MergedColumnParallelLinear(
            width, [m.heads * m.dim, m.kv_heads * m.dim,
                    m.kv_heads * m.vdim], dtype, seed_tag=tag)
        self.o_proj = RowParallelLinear(m.heads * m.vdim, width, dtype,
                                        seed_tag=tag + 3)
        self.q_norm, self.k_norm = RmsScale(m.dim), RmsScale(m.dim)
        # added to the scores of a head
        self.bias = _rows(_param(torch.zeros(m.heads // tp)), tp, r, m.heads)

    def forward(self, x, meta, cache) -> torch.Tensor:
        m = self.spec
        q, k, v = self.qkv.split(self.qkv(x))
        hybrid.norm_append(q, k, v, self.q_norm.w, self.k_norm.w, meta, cache,
                           self.eps)
        o = hybrid.sigmoid_attention(q, cache, meta, self.bias, m.chunk,
                                     m.scale, m.cap)
        return self.o_proj(o)

    def tensors(self, p: str):
        m, w = self.spec, self.width
        yield p + "q", (m.heads * m.dim, w), _part(self.qkv, 0)
        yield p + "k", (m.kv_heads * m.dim, w), _part(self.qkv, 1)
        yield p + "v", (m.kv_heads * m.vdim, w), _part(self.qkv, 2)
        yield p + "o", (w, m.heads * m.vdim), self.o_proj.load_full_weight
        yield from self.q_norm.tensors(p + "q.norm")
        yield from self.k_norm.tensors(p + "k.norm")
        yield p + "pb", (m.heads,), _put(self.bias, get_tp_size(),
                                         get_tp_rank())


class JoinedMixer(nn.Module):
    """A mixer that may have a dense feed-forward beside it, both reading one
    input and their outputs added: one product makes all projections of the
    input, one reduces the joined results [mixer | feed-forward], which adds
    them.  The activation rides along with the kernel that rotates."""

    def _join(self, width: int, parts: list, out: int, ff, dtype, tag: int,
              replicated: tuple = ()) -> None:
        if ff is not None and not isinstance(ff, SquaredRelu):
            raise ValueError("only a dense squared-ReLU feed-forward runs "
                             "beside a mixer")
        self.width, self.ff, self.out_size = width, ff, out
        hidden = [] if ff is None else [ff.ff]
        self.proj = MergedColumnParallelLinear(
            width, parts + hidden, dtype, seed_tag=tag,
            replicated=replicated, align=8)
        self.o_proj = MergedRowParallelLinear([out] + hidden, width, dtype,
                                              seed_tag=tag + len(parts) + 1)

    def enter(self, x: torch.Tensor):
        """The mixer's projections, its place in the joined results, these,
        and the activation to ride along (None: no feed-forward)."""
        parts = self.proj.split(self.proj(x))
        n = sum(self.o_proj.shard_sizes)
        joined = x.new_empty(x.shape[0], (n + 7) // 8 * 8)[:, :n]
        if self.ff is None:
            return parts, joined, joined, None
        m = self.o_proj.shard_sizes[0]
        return (parts[:-1], joined[:, :m], joined,
                hybrid.SideRelu(parts[-1], joined[:, m:]))

    def ff_tensors(self, p: str):
        if self.ff is not None:
            n, i = self.ff.ff, len(self.proj.out_sizes) - 1
            yield p + "up", (n, self.width), _part(self.proj, i)
            yield p + "down", (self.width, n), _part(self.o_proj, 1)

    def in_rows(self, name: str, i: int, order=None):
        """Tensor of the i-th projection; `order` of its rows."""
        yield name, (self.proj.out_sizes[i], self.width), \
            lambda t: self.proj.load_part(i, t if order is None else t[order])

    def out_columns(self, name: str, order=None):
        yield name, (self.width, self.out_size), \
            lambda t: self.o_proj.load_part(0, t if order is None
                                            else t[:, order])


class KeptWindowAttention(JoinedMixer):
    def __init__(self, spec: WindowAttention, width: int, eps: float, dtype,
                 tag: int, ff=None):
        super().__init__()
        self.spec, self.eps = spec, eps
        m = spec
        self._join(width, [m.heads * m.dim, m.kv_heads * m.dim,
                           m.kv_heads * m.vdim], m.heads * m.vdim, ff, dtype,
                   tag)
        buffer = lambda name, t: self.register_buffer(name, t,
                                                      persistent=False)
        buffer("freqs", frequencies(m.rot_dims, m.rot_base, m.stretch))
        buffer("turn", frequencies(m.vdim if m.turn_values else 0,
                                   m.rot_base))
        tp, r = get_tp_size(), get_tp_rank()
        self.sink = None if m.sink is None else _rows(_param(
            torch.full((m.heads // tp,), float(m.sink))), tp, r, m.heads)
        # normed queries and keys: a score is at most dim * |scale|
        self.bounded = m.qk_norm and m.dim * abs(m.scale) <= 40 \
            and abs(m.sink or 0.0) <= 40

    def forward(self, x, meta, cache) -> torch.Tensor:
        m = self.spec
        (q, k, v), out, joined, side = self.enter(x)
        hybrid.rope_norm_append(q, k, v, meta, self.freqs, self.turn, cache,
                                gain(m.stretch),
                                self.eps if m.qk_norm else None, side)
        hybrid.window_attention(out, q, cache, meta, self.turn, self.sink,
                                m.window, m.keep_first, m.scale,
                                self.bounded)
        return self.o_proj(joined)

    def tensors(self, p: str):
        m = self.spec
        qk = pair_order(m.dim, m.rot_dims, m.halves)
        v = pair_order(m.vdim, m.vdim, m.halves and m.turn_values)
        yield from self.in_rows(p + "q", 0, head_order(m.heads, m.dim, qk))
        yield from self.in_rows(p + "k", 1, head_order(m.kv_heads, m.dim, qk))
        yield from self.in_rows(p + "v", 2, head_order(m.kv_heads, m.vdim, v))
        yield from self.out_columns(p + "o", head_order(m.heads, m.vdim, v))


class WindowLatentAttention(JoinedMixer):
    def __init__(self, spec: LatentAttention, width: int, eps: float, dtype,
                 tag: int, ff=None):
        super().__init__()
        self.spec, self.eps = spec, eps
        m, tp, r = spec, get_tp_size(), get_tp_rank()
        self.owner = m.kv_from is None
        # q | latent, rotated key part (kept whole) | gate
        self._join(width, [m.heads * (m.dim + m.rot_dim)]
                   + [m.kv_rank + m.rot_dim] * self.owner
                   + [m.heads] * m.gate, m.heads * m.vdim, ff, dtype, tag,
                   replicated=(1,) * self.owner)
        # [rank, H * D]: rows of a head's key expansion are columns here, the
        # layout both the expansion and its absorption into q read
        d, e = m.heads * m.dim // tp, m.heads * m.vdim // tp
        uk = _init_weight(m.heads * m.dim, m.kv_rank, dtype, tag + 6)
        self.uk = _shard(
            _param(uk[r * d:(r + 1) * d].t().contiguous()), 1,
            [(r * d, d, 0)], (m.kv_rank, m.heads * m.dim))
        self.uv = _rows(_param(
            _init_weight(m.heads * m.vdim, m.kv_rank, dtype, tag + 7)
            [r * e:(r + 1) * e].contiguous()), tp, r, m.heads * m.vdim)
        self.kv_norm = RmsScale(m.kv_rank) if self.owner else None
        self.sink = _rows(_param(torch.zeros(m.heads // tp)), tp, r,
                          m.heads) if m.sink else None
        self.register_buffer(
            "freqs", frequencies(m.rot_dim, m.rot_base, m.stretch),
            persistent=False)

    def forward(self, x, meta, cache) -> torch.Tensor:
        m = self.spec
        heads = m.heads // get_tp_size()
        parts, out, joined, side = self.enter(x)
        kv = parts[1] if self.owner else None
        latent.rope_append(parts[0], kv,
                           self.kv_norm.w if self.owner else None, meta,
                           self.freqs, cache, heads, self.eps,
                           gain(m.stretch), side)
        latent.attention(parts[0], cache, meta, self.uk, self.uv, heads,
                         m.window, m.scale, self.sink,
                         parts[-1] if m.gate else None, out)
        return self.o_proj(joined)

    def tensors(self, p: str):
        m = self.spec
        tp, r = get_tp_size(), get_tp_rank()
        d = m.heads * m.dim // tp
        rotated = lambda first: pair_order(first + m.rot_dim, m.rot_dim,
                                           m.halves, first)
        yield from self.in_rows(p + "q", 0, head_order(
            m.heads, m.dim + m.rot_dim, rotated(m.dim)))
        if self.owner:
            yield from self.in_rows(p + "dkv", 1, rotated(m.kv_rank))
            yield from self.kv_norm.tensors(p + "dkv.norm")
        yield p + "uk", (m.heads * m.dim, m.kv_rank), \
            lambda t: self.uk.data.copy_(t[r * d:(r + 1) * d].t())
        yield p + "uv", (m.heads * m.vdim, m.kv_rank), _put(self.uv, tp, r)
        if m.sink:
            yield p + "sink", (m.heads,), _put(self.sink, tp, r)
        if m.gate:
            yield from self.in_rows(p + "g", 1 + self.owner)
        yield from self.out_columns(p + "o")


class LightningAttention(nn.Module):
    def __init__(self, spec: Lightning, width: int, eps: float, dtype,
                 tag: int):
        super().__init__()
        self.spec, self.width, self.eps = spec, width, eps
        m, tp, r = spec, get_tp_size(), get_tp_rank()
        d, e = m.heads * m.dim, m.heads * m.vdim
        self.proj = MergedColumnParallelLinear(width, [d, d, e, e], dtype,
                                               seed_tag=tag)
        self.o_proj = RowParallelLinear(e, width, dtype, seed_tag=tag + 4)
        self.norm = _rows(_param(torch.ones(e // tp)), tp, r, e)
        h = m.heads // tp
        self.decay = _rows(_param(torch.tensor(
            m.decay[r * h:(r + 1) * h], dtype=torch.float32)), tp, r, m.heads)

    def forward(self, x, meta, state) -> torch.Tensor:
        q, k, v, g = self.proj.split(self.proj(x))
        o = hybrid.lightning_mix(q, k, v, self.decay, state, meta)
        ss = None
        if get_tp_size() > 1:          # the norm spans the heads of all ranks
            ss = tensor_model_parallel_all_reduce(hybrid.row_squares(o))
        return self.o_proj(hybrid.rms_gate(o, g, self.norm, self.eps, ss,
                                           self.spec.heads * self.spec.vdim))

    def tensors(self, p: str):
        m, w = self.spec, self.width
        d, e = m.heads * m.dim, m.heads * m.vdim
        for i, (n, rows) in enumerate((("q", d), ("k", d), ("v", e),
                                       ("g", e))):
            yield p + n, (rows, w), _part(self.proj, i)
        yield p + "o", (w, e), self.o_proj.load_full_weight
        yield p + "norm", (e,), _put(self.norm, get_tp_size(), get_tp_rank())


MIXERS = {DiffAttention: WindowDiffAttention,
          GatedLinear: GatedLinearAttention,
          MatrixLSTM: MatrixMemoryLSTM,
          LatentAttention: WindowLatentAttention,
          Lightning: LightningAttention,
          SigmoidAttention: ChunkedSigmoidAttention,
          WindowAttention: KeptWindowAttention}
