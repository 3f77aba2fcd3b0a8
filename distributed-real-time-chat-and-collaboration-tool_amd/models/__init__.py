"""Model zoo: Llama-3 (8B/70B), Gemma-2B, Mixtral-8x7B (random-init bf16), and the designs with layers
of mixed kinds, Ralesun (latent attention + gated delta rule), Mebalorn (talking-heads attention +
minGRU), Nurilorn (capped attention with convolved projections + routed experts) and Garesun
(retention, matrix memory and attention over shared latents beside routed experts): random-init
presets and checkpoint folders."""
from __future__ import annotations

import os


from .checkpoint import read_safetensors
from .config import (GARESUN_5B, GARESUN_24B, GEMMA_2B, LLAMA3_8B, LLAMA3_70B, MEBALORN_2B, MEBALORN_8B, MIXTRAL_8X7B,
                     NURILORN_5B, NURILORN_24B, RALESUN_2B, RALESUN_8B, REGISTRY, TINY_GEMMA,
                     TINY_GARESUN, TINY_LLAMA, TINY_MEBALORN, TINY_MIXTRAL, TINY_NURILORN, TINY_RALESUN,
                     HybridConfig, ModelConfig, config_from_dict, get_config, load_config)
from .hybrid import HybridLM
from .transformer import DecodeMeta, PrefillMeta, TransformerLM


def build_model(cfg: ModelConfig | HybridConfig, device="cpu", *, tensors=None, **kw):
    """The model class of a configuration, with random weights or checkpoint ``tensors``."""
    if isinstance(cfg, HybridConfig):
        return HybridLM(cfg, device, tensors=tensors, **kw)
    if tensors is not None:
        raise ValueError(f"{cfg.name}: no checkpoint format for this family")
    return TransformerLM(cfg, device, **kw)


def load_model(name: str, device="cpu", *, max_position: int | None = None, **kw):
    """A registered model (random weights), or the checkpoint folder ``name``."""
    cfg = get_config(name)
    if name in REGISTRY:
        return build_model(cfg, device, **kw)
    if max_position is not None:
        cfg = cfg.replace(max_position=max_position)
    tensors = read_safetensors(os.path.join(name, "model.safetensors"))
    return build_model(cfg, device, tensors=tensors, **kw)


__all__ = ["GARESUN_5B", "GARESUN_24B", "TINY_GARESUN", "GEMMA_2B", "LLAMA3_8B", "LLAMA3_70B", "MEBALORN_2B", "MEBALORN_8B", "MIXTRAL_8X7B",
           "NURILORN_5B", "NURILORN_24B", "RALESUN_2B", "RALESUN_8B", "REGISTRY", "TINY_GEMMA",
           "TINY_LLAMA", "TINY_MEBALORN", "TINY_MIXTRAL", "TINY_NURILORN", "TINY_RALESUN", "HybridConfig",
           "HybridLM", "ModelConfig", "build_model", "config_from_dict", "get_config",
           "load_config", "load_model", "DecodeMeta", "PrefillMeta", "TransformerLM"]
