"""Mutusun: a decoder of chunked sigmoid attention without rotation, and dense
or expert feed-forwards.  Norms stand before and after every sublayer, a short
convolution over time is added to what a sublayer reads, the residual stream
is float, and a layer may run with another layer's tensors.

The configuration reader and tensor names live here; mixers, experts, caches
and kernels are shared parts (models.mixers, engine.kv_cache, ops).
"""

from __future__ import annotations

import os
from typing import List

import torch
from torch import nn

from hyperspot.engine.layer_spec import (Experts, HybridSpec, LayerSpec,
                                         SigmoidAttention, SquaredRelu,
                                         hybrid_spec)
from hyperspot.ops import hybrid
from hyperspot.parallel.layers import _init_weight

from .mixers import (MIXERS, ExpertMixture, InputConv, RmsScale,
                     SquaredReluMLP)

ARCHITECTURE = "Mutusun"


# ------------------------------------------------------------ configuration

def _mixer(kind: str, m: dict) -> SigmoidAttention:
    if kind != "attention":
        raise ValueError(f"{ARCHITECTURE}: unknown layer type {kind!r}")
    return SigmoidAttention(
        heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
        vdim=m["vdim"], scale=float(m["scale"]), cap=float(m["softcap"]),
        chunk=m["mask"]["size"])


def _feed_forward(mlp):
    if mlp is None:
        return None
    if mlp["kind"] == "dense":
        return SquaredRelu(mlp["ff"])
    if mlp["kind"] == "moe":
        r = mlp["router"]
        return Experts(experts=r["experts"], top=r["top"],
                       ff=mlp["expert"]["ff"], identity=r["identity"],
                       over_all=True, limit=float(mlp["expert"]["limit"]))
    raise ValueError(f"{ARCHITECTURE}: unknown feed-forward kind "
                     f"{mlp['kind']!r}")


def _spec(name: str, width: int, vocab: int, eps: float, taps: int,
          layers) -> HybridSpec:
    if taps < 1:
        raise ValueError(f"{ARCHITECTURE}: at least one tap")
    return hybrid_spec(name, ARCHITECTURE, width, vocab, eps, layers,
                       tie_embeddings=False, norm_params=width,
                       conv_taps=taps)


def spec_from_folder(cfg: dict, folder: str) -> HybridSpec:
    return _spec(os.path.basename(os.path.abspath(folder)), cfg["width"],
                 cfg["vocab"], float(cfg["norm"]["eps"]),
                 cfg["canon"]["taps"],
                 [LayerSpec(_mixer(e["type"], e["mixer"]),
                            _feed_forward(e.get("mlp")), e.get("weights_of"))
                  for e in cfg["layers"]])


def preset(name: str, width: int, vocab: int, heads: int, kv_heads: int,
           dim: int, chunk: int, ff: int, experts: Experts,
           layers: int, shared: int = 0) -> HybridSpec:
    """One layer with a dense feed-forward, the others with experts; the last
    `shared` of them run with the tensors of the second layer."""
    attn = SigmoidAttention(heads, kv_heads, dim, dim, dim ** -0.5, 50.0,
                            chunk)
    own = layers - shared
    return _spec(name, width, vocab, 1e-6, 4, [
        LayerSpec(attn, SquaredRelu(ff) if i == 0 else experts,
                  1 if i >= own else None) for i in range(layers)])


PRESETS = {
    # CPU / CI size, and one with the layer sizes of a real model
    "tiny-mutusun": lambda: preset(
        "tiny-mutusun", 96, 512, 4, 2, 24, 40, 160,
        Experts(5, 2, 48, identity=2, over_all=True, limit=5.0), 4, 1),
    "mutusun-16b": lambda: preset(
        "mutusun-16b", 2048, 102400, 16, 4, 128, 8192, 10944,
        Experts(64, 6, 1408, identity=16, over_all=True, limit=7.0), 28),
}


# -------------------------------------------------------------------- model

class MutusunLayer(nn.Module):
    def __init__(self, layer: LayerSpec, spec: HybridSpec, idx: int, dtype):
        super().__init__()
        w, taps, self.eps = spec.hidden_size, spec.conv_taps, spec.rms_eps
        tag = idx * 100
        norm = lambda: RmsScale(w, stored=1.0)
        self.norm1, self.norm1b = norm(), norm()
        self.conv1 = InputConv(w, taps, tag + 90)
        self.mix = MIXERS[type(layer.mixer)](layer.mixer, w, self.eps, dtype,
                                             tag=tag + 1)
        self.mlp = None
        if layer.ff is not None:
            self.norm2, self.norm2b = norm(), norm()
            self.conv2 = InputConv(w, taps, tag + 91)
            ff = ExpertMixture if isinstance(layer.ff, Experts) \
                else SquaredReluMLP
            self.mlp = ff(layer.ff, w, dtype, tag=tag + 50)

    def first_input(self, cache) -> hybrid.NextInput:
        return hybrid.NextInput(self.norm1.w, self.eps, self.conv1.w,
                                cache.tails[0])

    def forward(self, h, residual, meta, cache, nxt: hybrid.NextInput):
        """h is the mixer's input; returns the input that `nxt` makes of the
        residual after both sublayers were added."""
        h = self.mix(h, meta, cache.mixer)
        if self.mlp is None:
            return hybrid.add_rms_next(h, residual, self.norm1b.w, nxt, meta)
        h = hybrid.add_rms_next(
            h, residual, self.norm1b.w,
            hybrid.NextInput(self.norm2.w, self.eps, self.conv2.w,
                             cache.tails[1]), meta)
        return self.mlp.add_next(h, residual, self.norm2b, nxt, meta)

    def tensors(self, p: str):
        yield from self.norm1.tensors(p + "norm1")
        yield from self.norm1b.tensors(p + "norm1b")
        yield from self.conv1.tensors(p + "canon1")
        yield from self.mix.tensors(p + "mix.")
        if self.mlp is not None:
            yield from self.norm2.tensors(p + "norm2")
            yield from self.norm2b.tensors(p + "norm2b")
            yield from self.conv2.tensors(p + "canon2")
            yield from self.mlp.tensors(p + "mlp.")


class MutusunForCausalLM(nn.Module):
    def __init__(self, spec: HybridSpec, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        self.spec, self.dtype = spec, dtype
        table = lambda tag: nn.Parameter(
            _init_weight(spec.vocab_size, spec.hidden_size, dtype, tag),
            requires_grad=False)
        self.embed, self.head = table(900001), table(900002)
        # tensors once per owner, and the owner that every layer runs with
        self.owners = [i for i, layer in enumerate(spec.layers)
                       if layer.weights_of is None]
        self.blocks = nn.ModuleList([
            MutusunLayer(spec.layers[i], spec, i, dtype)
            for i in self.owners])
        self.runs = [self.owners.index(i if layer.weights_of is None
                                       else layer.weights_of)
                     for i, layer in enumerate(spec.layers)]
        self.final_norm = RmsScale(spec.hidden_size, stored=1.0)

    def forward(self, input_ids: torch.Tensor, meta,
                caches: List) -> torch.Tensor:
        """Returns logits [num_logit_rows, vocab]."""
        layers = [self.blocks[i] for i in self.runs]
        inputs = [layer.first_input(cache)
                  for layer, cache in zip(layers, caches)]
        inputs.append(hybrid.NextInput(self.final_norm.w, self.spec.rms_eps))
        residual = hybrid.embed_residual(self.embed, input_ids)
        h = hybrid.next_input(residual, inputs[0], meta, self.dtype)
        for layer, cache, nxt in zip(layers, caches, inputs[1:]):
            h = layer(h, residual, meta, cache, nxt)
            if meta.residual_trail is not None:
                meta.residual_trail.append(residual.clone())
        if meta.return_hidden:
            return h
        if meta.logits_indices is not None:
            h = h[meta.logits_indices]
        return h @ self.head.t()

    def named_tensors(self):
        """Checkpoint tensors of the design: (name, full shape, setter)."""
        for name, p in (("embed", self.embed), ("head", self.head)):
            yield name, tuple(p.shape), p.data.copy_
        for i, block in zip(self.owners, self.blocks):
            yield from block.tensors(f"l{i}.")
        yield from self.final_norm.tensors("final.norm")
