"""Radenex: a decoder of latent attention with sinks and output gates beside
windowed grouped-query attention that keeps the first tokens and turns its
values.  A layer has one norm; its mixer and its squared-ReLU feed-forward read
the same normed input and are added to a float residual at once.  A span of
layers may run several times with the same tensors.

The configuration reader and tensor names live here; mixers, caches and
kernels are shared parts (models.mixers, engine.kv_cache, ops).
"""

from __future__ import annotations

import os
from typing import List

import torch
from torch import nn

from hyperspot.engine.layer_spec import (UNBOUNDED, HybridSpec,
                                         LatentAttention, LayerSpec,
                                         SquaredRelu, WindowAttention,
                                         hybrid_spec, looped)
from hyperspot.engine.rotary import Yarn
from hyperspot.ops import hybrid
from hyperspot.parallel.layers import _init_weight

from .mixers import MIXERS, RmsScale

ARCHITECTURE = "Radenex"


# ------------------------------------------------------------ configuration

def _window(m: dict) -> WindowAttention:
    rot = m["rot"]
    return WindowAttention(
        heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
        vdim=m["vdim"], scale=float(m["scale"]),
        window=min(m["mask"]["size"], UNBOUNDED),
        keep_first=min(m["mask"]["keep_first"], UNBOUNDED),
        rot_dims=rot["dims"], rot_base=float(rot["base"]),
        stretch=float(rot["scaling"]["factor"]), halves=True, qk_norm=True,
        turn_values=True, sink=0.0)


def _latent(m: dict) -> LatentAttention:
    rot = m["rot"]
    if rot["dims"] != m["rot_dim"]:
        raise ValueError(f"{ARCHITECTURE}: rot.dims must equal rot_dim")
    return LatentAttention(
        heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"], vdim=m["vdim"],
        kv_rank=m["kv_rank"], scale=float(m["scale"]), window=UNBOUNDED,
        rot_base=float(rot["base"]), halves=True, sink=True, gate=True,
        stretch=Yarn(**{k: float(rot["scaling"][k])
                        for k in ("factor", "original", "fast", "slow")}))


_MIXERS = {"attention": _window, "latent_attention": _latent}


def _layer(entry: dict) -> LayerSpec:
    if entry["type"] not in _MIXERS:
        raise ValueError(f"{ARCHITECTURE}: unknown layer type "
                         f"{entry['type']!r}")
    mlp = entry.get("mlp")
    if mlp is not None and mlp["kind"] != "dense":
        raise ValueError(f"{ARCHITECTURE}: unknown feed-forward kind "
                         f"{mlp['kind']!r}")
    return LayerSpec(_MIXERS[entry["type"]](entry["mixer"]),
                     None if mlp is None else SquaredRelu(mlp["ff"]))


def _spec(name: str, width: int, vocab: int, eps: float,
          layers) -> HybridSpec:
    return hybrid_spec(name, ARCHITECTURE, width, vocab, eps, layers,
                       tie_embeddings=False, norm_params=width, norms=1,
                       parallel=True)


def spec_from_folder(cfg: dict, folder: str) -> HybridSpec:
    layers = [_layer(e) for e in cfg["layers"]]
    loop = cfg.get("loop")
    if loop is not None:
        layers = looped(layers, loop["start"], loop["stop"], loop["times"])
    return _spec(os.path.basename(os.path.abspath(folder)), cfg["width"],
                 cfg["vocab"], float(cfg["norm"]["eps"]), layers)


def preset(name: str, width: int, vocab: int, heads: int, kv_heads: int,
           dim: int, window: int, keep_first: int, latent_heads: int,
           latent_dim: int, rot_dim: int, kv_rank: int, ff: int, layers: int,
           loop: tuple = (0, 0, 1)) -> HybridSpec:
    """Windowed and latent attention in turn."""
    kinds = (WindowAttention(heads, kv_heads, dim, dim, dim ** -0.5, window,
                             dim // 2, 10000.0, keep_first, 4.0, True, True,
                             True, 0.0),
             LatentAttention(latent_heads, latent_dim, rot_dim, latent_dim,
                             kv_rank, (latent_dim + rot_dim) ** -0.5,
                             UNBOUNDED, 1e6, None,
                             Yarn(8.0, 4096.0, 32.0, 1.0), True, True, True))
    return _spec(name, width, vocab, 1e-6, looped(
        [LayerSpec(kinds[i % 2], SquaredRelu(ff)) for i in range(layers)],
        *loop))


PRESETS = {
    # CPU / CI size, and one with the layer sizes of a real model
    "tiny-radenex": lambda: preset("tiny-radenex", 96, 512, 4, 2, 24, 20, 3,
                                   3, 24, 16, 40, 160, 4, (1, 3, 2)),
    "radenex-8b": lambda: preset("radenex-8b", 4096, 102400, 32, 8, 128, 4096,
                                 4, 32, 128, 64, 512, 21504, 32),
}


# -------------------------------------------------------------------- model

class RadenexLayer(nn.Module):
    def __init__(self, layer: LayerSpec, spec: HybridSpec, idx: int, dtype):
        super().__init__()
        self.norm = RmsScale(spec.hidden_size)
        self.mix = MIXERS[type(layer.mixer)](
            layer.mixer, spec.hidden_size, spec.rms_eps, dtype,
            tag=idx * 100 + 1, ff=layer.ff)

    def tensors(self, p: str):
        yield from self.norm.tensors(p + "norm1")
        yield from self.mix.tensors(p + "mix.")
        yield from self.mix.ff_tensors(p + "mlp.")


class RadenexForCausalLM(nn.Module):
    def __init__(self, spec: HybridSpec, dtype: torch.dtype = torch.bfloat16):
        super().__init__()
        self.spec, self.dtype = spec, dtype
        table = lambda tag: nn.Parameter(
            _init_weight(spec.vocab_size, spec.hidden_size, dtype, tag),
            requires_grad=False)
        self.embed, self.head = table(900001), table(900002)
        # tensors once per layer of the configuration, and for every run the
        # layer whose tensors it uses
        owners = [i for i, layer in enumerate(spec.layers)
                  if layer.weights_of is None]
        self.blocks = nn.ModuleList([
            RadenexLayer(spec.layers[i], spec, n, dtype)
            for n, i in enumerate(owners)])
        self.runs = [owners.index(i if layer.weights_of is None
                                  else layer.weights_of)
                     for i, layer in enumerate(spec.layers)]
        self.final_norm = RmsScale(spec.hidden_size)

    def forward(self, input_ids: torch.Tensor, meta,
                caches: List) -> torch.Tensor:
        """Returns logits [num_logit_rows, vocab]."""
        layers = [self.blocks[i] for i in self.runs]
        inputs = [hybrid.NextInput(norm.w, self.spec.rms_eps)
                  for norm in [x.norm for x in layers] + [self.final_norm]]
        residual = hybrid.embed_residual(self.embed, input_ids)
        h = hybrid.next_input(residual, inputs[0], meta, self.dtype)
        for layer, cache, nxt in zip(layers, caches, inputs[1:]):
            h = hybrid.add_next(layer.mix(h, meta, cache), residual, nxt,
                                meta)
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
        for i, block in enumerate(self.blocks):
            yield from block.tensors(f"l{i}.")
        yield from self.final_norm.tensors("final.norm")
