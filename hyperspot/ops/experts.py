"""Mixture of gated experts with an optional shared expert.

A GPU tensor runs the gfx950 kernels of csrc/experts.hip (and, for large
steps, the grouped products of csrc/moe.hip), a CPU tensor the PyTorch
reference.  Weights: router [E + I + 1, W] (after the experts come I identity
outputs, whose expert is the input itself, then the shared expert's gate, which
is absent without one), up [E, 2F, W] with gate rows first, down [E, W, F], the
shared pair likewise with one expert.  `Rules` says how choices are weighted
and which activation the experts have.

Three ways on the GPU, chosen by shapes only so that a captured graph keeps
its choice:

  rows      bf16, few rows per expert: tiles of 16 to 64 rows; the weights
            stream from memory once; the shared expert is one more expert
            that every token has chosen.
  tiles     bf16, many rows per expert: the 256-row tiles of csrc/moe.hip,
            the shared expert as plain products.
  general   any sizes, bf16 or float.
"""

from __future__ import annotations

from typing import NamedTuple, Optional

import torch

from . import MOE_BM, _moe_splitk, _native, silu_mul, torch_ref
from .hybrid import NextInput, _conv_ref, clamped_glu, gate_projection

TILES_FROM = 96        # mean rows per expert from which 256-row tiles pay


class Rules(NamedTuple):
    """Routing and activation.  With a correction [E + I] float the weights
    are the softmax over all outputs and the correction is added for the
    choice only; without, they are the softmax over the chosen.  With a limit
    experts are clamped gated units (hybrid.clamped_glu), otherwise
    silu(gate) * up."""

    correction: Optional[torch.Tensor] = None
    identity: int = 0
    limit: Optional[float] = None
    # this rank adds the identity experts' part
    identity_here: bool = True


def mixture_add_rms(x, router, up, down, shared_up, shared_down, top: int,
                    residual, w, eps: float,
                    rules: Rules = Rules()) -> torch.Tensor:
    """residual += rms(mixture(x)) * w in place; the residual in x's type."""
    args = (x, router, up, down, shared_up, shared_down, top, rules)
    if not x.is_cuda:
        residual += torch_ref.rms_scale(torch_ref.mixture(*args), w, eps)
        return residual.to(x.dtype)
    out = residual if x.dtype == torch.float32 else torch.empty_like(x)
    _native().experts_sum(out, *_run(*args), _identity(x, rules), residual, w,
                          eps)
    return out


def mixture_add_next(x, router, up, down, shared_up, shared_down, top: int,
                     rules: Rules, residual, w, nxt: NextInput,
                     meta) -> torch.Tensor:
    """residual += rms(mixture(x)) * w in place; returns the next sublayer's
    input in x's type."""
    args = (x, router, up, down, shared_up, shared_down, top, rules)
    if not x.is_cuda:
        residual += torch_ref.rms_scale(torch_ref.mixture(*args), w, nxt.eps)
        h = torch_ref.rms_scale(residual, nxt.w, nxt.eps).to(x.dtype)
        return _conv_ref(h, nxt, meta)
    h = torch.empty_like(x)
    _native().experts_sum_next(h, *_run(*args), _identity(x, rules), residual,
                               w, nxt.w, nxt.eps, *nxt.row_args(meta))
    return nxt.finish(h, meta)


def mixture(x, router, up, down, shared_up, shared_down, top: int,
            rules: Rules = Rules()) -> torch.Tensor:
    """The weighted sum itself, in x's type."""
    args = (x, router, up, down, shared_up, shared_down, top, rules)
    if not x.is_cuda:
        return torch_ref.mixture(*args).to(x.dtype)
    out = torch.empty_like(x)
    _native().experts_sum(out, *_run(*args), _identity(x, rules), None, None,
                          0.0)
    return out


def _identity(x, rules: Rules):
    return x if rules.identity and rules.identity_here else None


def _run(x, router, up, down, shared_up, shared_down, top, rules):
    """(y, place, weight, shared): expert outputs y [P, W], the row of every
    choice `place` [T, n] (-1: an identity expert), choice weights
    [T, top + 1 or top], and the shared expert's own rows if they are not in
    y."""
    n = _native()
    T, W = x.shape
    E, F = up.shape[0], down.shape[2]
    has = shared_up is not None
    Fs = shared_down.shape[2] if has else 0
    i32 = lambda *s: torch.empty(*s, dtype=torch.int32, device=x.device)
    logits = gate_projection(x, router)
    weight = torch.empty(T, top + has, dtype=torch.float32, device=x.device)
    bf = x.dtype == torch.bfloat16
    mean = T * top / (E + rules.identity)
    act = silu_mul if rules.limit is None \
        else lambda h: clamped_glu(h, rules.limit)
    route = (E, top, rules.correction, rules.identity)
    if bf and mean >= TILES_FROM and W % 128 == 0 and F % 128 == 0:
        ids = i32(T, top)
        n.experts_route(weight, ids, logits, *route)
        y, place = _tiles(n, x, up, down, ids, act)
        shared = act(x @ shared_up[0].t()) @ shared_down[0].t() \
            if has else None
        return y, place, weight, shared
    fast = bf and W % 8 == 0 and F % 8 == 0 and Fs % 8 == 0
    bm = 1 if not fast else 16 if mean <= 16 else 32 if mean <= 32 else 64
    pairs, kinds = T * (top + has), E + has
    tiles = min(pairs, (pairs + kinds * (bm - 1)) // bm)
    ids, place = i32(T, top + has), i32(T, top + has)
    order, expert = i32(tiles * bm), i32(tiles)
    n.experts_route_sort(weight, ids, place, order, expert, logits, bm,
                         *route)
    h = torch.empty(tiles * bm, max(F, Fs), dtype=x.dtype, device=x.device)
    y = torch.empty(tiles * bm, W, dtype=x.dtype, device=x.device)
    n.experts_up(h, x, up, shared_up, order, expert, top + has, rules.limit,
                 bm)
    n.experts_down(y, h, down, shared_down, order, expert, bm)
    return y, place, weight, None


def _tiles(n, x, up, down, ids, act):
    T, W = x.shape
    E, top, F2 = up.shape[0], ids.shape[1], up.shape[1]
    tiles = (T * top + E * (MOE_BM - 1) + MOE_BM - 1) // MOE_BM
    P, dev = tiles * MOE_BM, x.device
    i32 = lambda *s: torch.empty(*s, dtype=torch.int32, device=dev)
    order, expert, place = i32(P), i32(tiles), i32(T * top)
    n.experts_sort(order, expert, place, ids.view(-1), E, MOE_BM)
    h = torch.empty(P, F2, dtype=x.dtype, device=dev)
    s, ws = _moe_splitk(tiles * (F2 // 128), W // 64, P * F2, dev)
    n.moe_gemm(h, x, up, order, expert, top, s, ws)
    a = act(h)
    y = torch.empty(P, W, dtype=x.dtype, device=dev)
    s, ws = _moe_splitk(tiles * (W // 128), F2 // 128, P * W, dev)
    n.moe_gemm(y, a, down, order, expert, 0, s, ws)
    return y, place.view(T, top)
