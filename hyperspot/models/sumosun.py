"""Sumosun: a decoder whose layers mix windowed differential attention, gated
linear attention and matrix LSTMs, with dynamic-tanh norms before and after
every sublayer and a float residual stream.

The configuration reader and tensor names live here; mixers, caches and
kernels are shared parts (models.mixers, engine.kv_cache, ops.hybrid).
"""

from __future__ import annotations

import os
from typing import List

import torch
from torch import nn

from hyperspot.engine.layer_spec import (DiffAttention, GatedLinear,
                                         HybridSpec, LayerSpec, MatrixLSTM,
                                         hybrid_spec)
from hyperspot.ops import hybrid
from hyperspot.parallel.layers import _init_weight

from .mixers import MIXERS, DynamicTanh, GatedGelu

ARCHITECTURE = "Sumosun"


# ------------------------------------------------------------ configuration

def _mixer(kind: str, m: dict, rank: int):
    if kind == "attention":
        return DiffAttention(
            heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
            vdim=m["vdim"], scale=float(m["scale"]),
            window=m["mask"]["size"], rot_dims=m["rot"]["dims"],
            rot_base=float(m["rot"]["base"]), diff=float(m["diff"]))
    if kind == "gla":
        return GatedLinear(heads=m["heads"], dim=m["dim"], vdim=m["vdim"],
                           tau=float(m["tau"]), rank=rank)
    if kind == "mlstm":
        return MatrixLSTM(heads=m["heads"], dim=m["dim"], vdim=m["vdim"],
                          gate_cap=float(m["gate_cap"]))
    raise ValueError(f"{ARCHITECTURE}: unknown layer type {kind!r}")


def spec_from_config(cfg: dict, shapes: dict, name: str) -> HybridSpec:
    """`shapes` maps tensor names to shapes: the inner size of a decay
    projection is given by its tensor only."""
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        rank = shapes[f"l{i}.mix.a1"][0] if entry["type"] == "gla" else 0
        mlp = entry.get("mlp")
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"{ARCHITECTURE}: unknown feed-forward kind "
                             f"{mlp['kind']!r}")
        layers.append(LayerSpec(_mixer(entry["type"], entry["mixer"], rank),
                                None if mlp is None else mlp["ff"]))
    return hybrid_spec(name, ARCHITECTURE, cfg["width"], cfg["vocab"],
                       float(cfg["norm"]["eps"]), layers,
                       norm_params=2 * cfg["width"] + 1)


def preset(name: str, width: int, vocab: int, ff: int, heads: int,
           kv_heads: int, dim: int, window: int, periods: int,
           state_heads: int) -> HybridSpec:
    """Repeats of (attention + ff, mLSTM, GLA + ff)."""
    attn = DiffAttention(heads, kv_heads, dim, 2 * dim, dim ** -0.5, window,
                         rot_dims=dim // 2, rot_base=100000.0, diff=0.45)
    lstm = MatrixLSTM(state_heads, dim, 2 * dim, gate_cap=12.0)
    gla = GatedLinear(state_heads, dim, 2 * dim, tau=8.0, rank=24)
    layers = [LayerSpec(attn, ff), LayerSpec(lstm), LayerSpec(gla, ff)]
    return hybrid_spec(name, ARCHITECTURE, width, vocab, 1e-5,
                       layers * periods, norm_params=2 * width + 1)


PRESETS = {
    # CPU / CI size, and one with the layer sizes of a real model
    "tiny-sumosun": lambda: preset("tiny-sumosun", 192, 512, 288, 4, 2, 24,
                                   20, 1, 2),
    "sumosun-3b": lambda: preset("sumosun-3b", 4096, 128256, 14336, 32, 8,
                                 64, 1024, 4, 16),
}


# -------------------------------------------------------------------- model

class SumosunLayer(nn.Module):
    def __init__(self, layer: LayerSpec, spec: HybridSpec, idx: int, dtype):
        super().__init__()
        w = spec.hidden_size
        self.norm1, self.norm1b = DynamicTanh(w), DynamicTanh(w)
        self.mix = MIXERS[type(layer.mixer)](layer.mixer, w, spec.rms_eps,
                                             dtype, tag=idx * 100 + 1)
        self.mlp = None
        if layer.ff is not None:
            self.norm2, self.norm2b = DynamicTanh(w), DynamicTanh(w)
            self.mlp = GatedGelu(w, layer.ff, dtype, tag=idx * 100 + 50)

    def forward(self, h, residual, meta, cache, next_norm):
        """h is norm1(residual); returns next_norm(residual) after both
        sublayers were added (each post-norm, add and following pre-norm is
        one kernel)."""
        h = self.mix(h, meta, cache)
        if self.mlp is None:
            return hybrid.add_dyt(h, residual, self.norm1b.args,
                                  next_norm.args)
        h = hybrid.add_dyt(h, residual, self.norm1b.args, self.norm2.args)
        h = self.mlp(h)
        return hybrid.add_dyt(h, residual, self.norm2b.args, next_norm.args)

    def tensors(self, p: str):
        yield from self.norm1.tensors(p + "norm1")
        yield from self.norm1b.tensors(p + "norm1b")
        yield from self.mix.tensors(p + "mix.")
        if self.mlp is not None:
            yield from self.norm2.tensors(p + "norm2")
            yield from self.norm2b.tensors(p + "norm2b")
            yield from self.mlp.tensors(p + "mlp.")


class SumosunForCausalLM(nn.Module):
    def __init__(self, spec: HybridSpec, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        self.spec, self.dtype = spec, dtype
        self.embed = nn.Parameter(
            _init_weight(spec.vocab_size, spec.hidden_size, dtype, 900001),
            requires_grad=False)
        self.layers = nn.ModuleList([
            SumosunLayer(layer, spec, i, dtype)
            for i, layer in enumerate(spec.layers)])
        self.final_norm = DynamicTanh(spec.hidden_size)

    def forward(self, input_ids: torch.Tensor, meta,
                caches: List) -> torch.Tensor:
        """Returns logits [num_logit_rows, vocab]."""
        norms = [layer.norm1 for layer in self.layers] + [self.final_norm]
        h, residual = hybrid.embed_dyt(self.embed, input_ids, norms[0].args)
        for layer, cache, nxt in zip(self.layers, caches, norms[1:]):
            h = layer(h, residual, meta, cache, nxt)
            if meta.residual_trail is not None:
                meta.residual_trail.append(residual.clone())
        if meta.return_hidden:
            return h
        if meta.logits_indices is not None:
            h = h[meta.logits_indices]
        return h @ self.embed.t()

    def named_tensors(self):
        """Checkpoint tensors of the design: (name, full shape, setter)."""
        yield "embed", tuple(self.embed.shape), self.embed.data.copy_
        for i, layer in enumerate(self.layers):
            yield from layer.tensors(f"l{i}.")
        yield from self.final_norm.tensors("final.norm")


def spec_from_folder(cfg: dict, folder: str) -> HybridSpec:
    from hyperspot.engine.checkpoint import tensor_shapes
    return spec_from_config(cfg, tensor_shapes(folder),
                            os.path.basename(os.path.abspath(folder)))
