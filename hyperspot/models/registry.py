"""Model registry: spec -> model class, and model folder -> spec (the
in-engine half; the tenant-facing model-registry module with canonical
`{provider}::{model}` ids lives in the C++ host plane, reference
modules/model-registry/docs/PRD.md)."""

from __future__ import annotations

import json
import os

import torch

from hyperspot.engine.config import ModelSpec, get_model_spec

from . import mutusun, radenex, sumosun, tefezen

# config.json "architecture" -> (configuration reader, model class)
DESIGNS = {
    sumosun.ARCHITECTURE: (sumosun.spec_from_folder,
                           sumosun.SumosunForCausalLM),
    tefezen.ARCHITECTURE: (tefezen.spec_from_folder,
                           tefezen.TefezenForCausalLM),
    mutusun.ARCHITECTURE: (mutusun.spec_from_folder,
                           mutusun.MutusunForCausalLM),
    radenex.ARCHITECTURE: (radenex.spec_from_folder,
                           radenex.RadenexForCausalLM),
}

# presets of the designs (random-init), by canonical id
DESIGN_PRESETS = {**sumosun.PRESETS, **tefezen.PRESETS, **mutusun.PRESETS,
                  **radenex.PRESETS}


def spec_from_folder(folder: str) -> ModelSpec:
    path = os.path.join(folder, "config.json")
    with open(path) as f:
        cfg = json.load(f)
    arch = cfg.get("architecture")
    if arch not in DESIGNS:
        raise KeyError(f"{path}: unknown architecture {arch!r} "
                       f"(have: {sorted(DESIGNS)})")
    return DESIGNS[arch][0](cfg, folder)


def build_model(spec_or_name, dtype: torch.dtype = torch.bfloat16):
    from .llama import LlamaForCausalLM
    from .mixtral import MixtralForCausalLM
    spec = spec_or_name if isinstance(spec_or_name, ModelSpec) \
        else get_model_spec(spec_or_name)
    if spec.is_hybrid:
        cls = DESIGNS[spec.architecture][1]
    else:
        cls = MixtralForCausalLM if spec.is_moe else LlamaForCausalLM
    return cls(spec, dtype=dtype)
