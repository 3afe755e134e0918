"""Model families: which config class, module, weight names and step runner serve a ``config.json``.

HF configs carry ``model_type`` and map onto ``CausalLM``; native designs carry ``architecture``. Everything
that loads, serves or saves a model goes through the lookups here, so a design added to ``FAMILIES`` is
available to all of them.
"""
from __future__ import annotations

import dataclasses
import json
import os
from typing import Callable


@dataclasses.dataclass(frozen=True)
class Family:
    """``kernels``: the ``csrc/kernels`` sources a fresh checkout needs to run the family's step."""
    name: str
    read_config: Callable
    build: Callable            # (cfg, device, dtype, seed) -> module
    to_native: Callable        # (checkpoint tensors, cfg) -> module state
    from_native: Callable
    runner: Callable           # () -> StepRunner class
    kernels: tuple = ()
    with_shapes: Callable | None = None  # (cfg, {checkpoint tensor: shape}) -> cfg with the sizes only they give


def _megusun() -> Family:
    from . import megusun
    from .hybrid_lm import build_hybrid

    def runner():
        from ..engine.hybrid_runner import HybridRunner
        return HybridRunner
    return Family("megusun", megusun.read_config, build_hybrid, megusun.to_native, megusun.from_native, runner,
                  ("rms_shift", "gated_scan", "diff_attn", "moe", "act_rows", "gemv", "skinny_mfma"))


def _rezusun() -> Family:
    from . import rezusun
    from .hybrid_lm import build_hybrid

    def runner():
        from ..engine.hybrid_runner import HybridRunner
        return HybridRunner
    return Family("rezusun", rezusun.read_config, build_hybrid, rezusun.to_native, rezusun.from_native, runner,
                  ("norm_residual", "delta_rule", "delta_chunk", "latent_attn", "latent_mfma", "act_rows", "gemv", "skinny_mfma"),
                  rezusun.with_shapes)


def _begopel() -> Family:
    from . import begopel
    from .hybrid_lm import build_hybrid

    def runner():
        from ..engine.hybrid_runner import HybridRunner
        return HybridRunner
    return Family("begopel", begopel.read_config, build_hybrid, begopel.to_native, begopel.from_native, runner,
                  ("norm_residual", "delta_rule", "delta_chunk", "ssd_chunk", "biased_attn", "act_rows", "gemv", "skinny_mfma"),
                  begopel.with_shapes)


def _gibipel() -> Family:
    from . import gibipel
    from .hybrid_lm import build_hybrid

    def runner():
        from ..engine.hybrid_runner import HybridRunner
        return HybridRunner
    return Family("gibipel", gibipel.read_config, build_hybrid, gibipel.to_native, gibipel.from_native, runner,
                  ("norm_residual", "pooled_attn", "matrix_memory", "side_step", "moe", "act_rows", "gemv", "skinny_mfma"))


def _causal_lm() -> Family:
    from .causal_lm import build_causal_lm
    from .config import LMConfig
    from .hf_convert import hf_to_native, native_to_hf

    def runner():
        from ..engine.runner import ModelRunner
        return ModelRunner
    return Family("causal_lm", LMConfig.read_hf, build_causal_lm, hf_to_native, native_to_hf, runner)


FAMILIES = {"Megusun": _megusun, "Rezusun": _rezusun, "Begopel": _begopel, "Gibipel": _gibipel}   # config.json "architecture" -> family


def family_of_dict(cfg: dict) -> Family:
    arch = cfg.get("architecture")
    if arch is None:
        return _causal_lm()
    if arch not in FAMILIES:
        from .config import UnsupportedModel
        raise UnsupportedModel(arch)
    return FAMILIES[arch]()


def family_of(cfg) -> Family:
    """Family of a parsed config (``LMConfig`` / ``HybridConfig``)."""
    for make in FAMILIES.values():
        f = make()
        if f.name == cfg.arch:
            return f
    return _causal_lm()


def require_causal_lm(cfg, what: str):
    """``cfg`` if it is an HF family's ``LMConfig``; the paths that handle those alone name the limit."""
    from .config import LMConfig
    if not isinstance(cfg, LMConfig):
        raise NotImplementedError(f"{what} supports the HF causal-LM families, not {cfg.arch} (which serves on one GPU)")
    return cfg


def read_dict(path: str) -> dict:
    with open(os.path.join(path, "config.json")) as f:
        return json.load(f)


__all__ = ["Family", "FAMILIES", "family_of", "family_of_dict", "read_dict", "require_causal_lm"]
