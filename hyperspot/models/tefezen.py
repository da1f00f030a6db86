"""Tefezen: a decoder whose layers mix windowed latent attention and lightning
attention with mixtures of experts.  Norms follow the sublayers only, the
residual stream is float, every layer also takes an input of the token's own,
and a latent-attention layer may use an earlier layer's latents.

The configuration reader and tensor names live here; mixers, experts, caches
and kernels are shared parts (models.mixers, engine.kv_cache, ops).
"""

from __future__ import annotations

import os
from typing import List

import torch
from torch import nn

from hyperspot.engine.layer_spec import (Experts, HybridSpec, LatentAttention,
                                         LayerSpec, Lightning, hybrid_spec)
from hyperspot.ops import hybrid
from hyperspot.parallel.layers import _init_weight

from .mixers import MIXERS, ExpertMixture, RmsScale, TokenSide

ARCHITECTURE = "Tefezen"


# ------------------------------------------------------------ configuration

def _mixer(kind: str, m: dict):
    if kind == "latent_attention":
        if m["rot"]["dims"] != m["rot_dim"]:
            raise ValueError(f"{ARCHITECTURE}: rot.dims must equal rot_dim")
        return LatentAttention(
            heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"],
            vdim=m["vdim"], kv_rank=m["kv_rank"], scale=float(m["scale"]),
            window=m["mask"]["size"], rot_base=float(m["rot"]["base"]),
            kv_from=m.get("kv_from"))
    if kind == "lightning":
        return Lightning(heads=m["heads"], dim=m["dim"], vdim=m["vdim"],
                         decay=tuple(float(x) for x in m["decay"]))
    raise ValueError(f"{ARCHITECTURE}: unknown layer type {kind!r}")


def _feed_forward(mlp):
    if mlp is None:
        return None
    if mlp["kind"] != "moe":
        raise ValueError(f"{ARCHITECTURE}: unknown feed-forward kind "
                         f"{mlp['kind']!r}")
    shared = mlp.get("shared")
    return Experts(experts=mlp["router"]["experts"], top=mlp["router"]["top"],
                   ff=mlp["expert"]["ff"],
                   shared=None if shared is None else shared["ff"])


def _spec(name: str, width: int, vocab: int, eps: float, embed_scale: float,
          side_dim: int, layers) -> HybridSpec:
    return hybrid_spec(name, ARCHITECTURE, width, vocab, eps, layers,
                       tie_embeddings=False, norm_params=width, norms=1,
                       embed_scale=embed_scale, side_dim=side_dim)


def spec_from_folder(cfg: dict, folder: str) -> HybridSpec:
    return _spec(os.path.basename(os.path.abspath(folder)), cfg["width"],
                 cfg["vocab"], float(cfg["norm"]["eps"]),
                 float(cfg["embedding"]["scale"]), cfg["token_side"]["dim"],
                 [LayerSpec(_mixer(e["type"], e["mixer"]),
                            _feed_forward(e.get("mlp")))
                  for e in cfg["layers"]])


def preset(name: str, width: int, vocab: int, heads: int, dim: int,
           rot_dim: int, kv_rank: int, window: int, state_heads: int,
           state_dim: int, experts: Experts, side_dim: int,
           periods: int) -> HybridSpec:
    """Repeats of (lightning, latent, lightning, latent over the second
    layer's latents), experts in every layer."""
    fast = Lightning(state_heads, state_dim, state_dim, tuple(
        1.0 - 2.0 ** (-1 - 8 * i / state_heads) for i in range(state_heads)))
    layers = []
    for p in range(periods):
        for kv_from in (None, 4 * p + 1):
            layers += [LayerSpec(fast, experts), LayerSpec(LatentAttention(
                heads, dim, rot_dim, dim, kv_rank, (dim + rot_dim) ** -0.5,
                window, 10000.0, kv_from), experts)]
    return _spec(name, width, vocab, 1e-6, width ** 0.5, side_dim, layers)


PRESETS = {
    # CPU / CI size, and one with the layer sizes of a real model
    "tiny-tefezen": lambda: preset("tiny-tefezen", 96, 512, 3, 24, 16, 40, 20,
                                   2, 24, Experts(5, 2, 48, 64), 8, 1),
    "tefezen-16b": lambda: preset("tefezen-16b", 2048, 102400, 16, 128, 64,
                                  512, 4096, 16, 128, Experts(64, 6, 1408,
                                                              2816), 128, 6),
}


# -------------------------------------------------------------------- model

class TefezenLayer(nn.Module):
    def __init__(self, layer: LayerSpec, spec: HybridSpec, idx: int, dtype):
        super().__init__()
        w, self.eps = spec.hidden_size, spec.rms_eps
        self.mix = MIXERS[type(layer.mixer)](layer.mixer, w, self.eps, dtype,
                                             tag=idx * 100 + 1)
        self.norm1 = RmsScale(w, stored=1.0)
        self.mlp = None
        if layer.ff is not None:
            self.mlp = ExpertMixture(layer.ff, w, dtype, tag=idx * 100 + 50)
            self.norm2 = RmsScale(w, stored=1.0)
        self.side = TokenSide(w, spec.side_dim, idx * spec.side_dim, dtype,
                              tag=idx * 100 + 80)

    def forward(self, x, residual, table, ids, meta, cache):
        """x is the residual in the model's element type; returns the same
        after both sublayers and the token's input were added."""
        x = hybrid.add_rms(self.mix(x, meta, cache), residual, self.norm1.w,
                           self.eps, x.dtype)
        if self.mlp is not None:
            x = self.mlp.add_normed(x, residual, self.norm2, self.eps)
        return self.side.add(x, residual, table, ids, self.eps)

    def tensors(self, p: str):
        yield from self.mix.tensors(p + "mix.")
        yield from self.norm1.tensors(p + "norm1")
        if self.mlp is not None:
            yield from self.mlp.tensors(p + "mlp.")
            yield from self.norm2.tensors(p + "norm2")
        yield from self.side.tensors(p + "side.")


class TefezenForCausalLM(nn.Module):
    def __init__(self, spec: HybridSpec, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        self.spec, self.dtype = spec, dtype
        table = lambda cols, tag: nn.Parameter(
            _init_weight(spec.vocab_size, cols, dtype, tag),
            requires_grad=False)
        self.embed = table(spec.hidden_size, 900001)
        self.head = table(spec.hidden_size, 900002)
        self.side_embed = table(spec.side_dim * len(spec.layers), 900003)
        self.layers = nn.ModuleList([
            TefezenLayer(layer, spec, i, dtype)
            for i, layer in enumerate(spec.layers)])
        self.final_norm = RmsScale(spec.hidden_size, stored=1.0)

    def forward(self, input_ids: torch.Tensor, meta,
                caches: List) -> torch.Tensor:
        """Returns logits [num_logit_rows, vocab]."""
        x, residual = hybrid.embed_scaled(self.embed, input_ids,
                                          self.spec.embed_scale)
        for layer, cache in zip(self.layers, caches):
            x = layer(x, residual, self.side_embed, input_ids, meta, cache)
            if meta.residual_trail is not None:
                meta.residual_trail.append(residual.clone())
        if meta.logits_indices is not None and not meta.return_hidden:
            residual = residual[meta.logits_indices]
        h = hybrid.rms_scale(residual, self.final_norm.w, self.spec.rms_eps,
                             self.dtype)
        return h if meta.return_hidden else h @ self.head.t()

    def named_tensors(self):
        """Checkpoint tensors of the design: (name, full shape, setter)."""
        for name, p in (("embed", self.embed), ("head", self.head),
                        ("side.embed", self.side_embed)):
            yield name, tuple(p.shape), p.data.copy_
        for i, layer in enumerate(self.layers):
            yield from layer.tensors(f"l{i}.")
        yield from self.final_norm.tensors("final.norm")
