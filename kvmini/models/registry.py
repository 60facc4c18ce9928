"""Model families the engine serves: how a name or a checkpoint directory becomes a configuration, where its weights come
from, and which runner executes it.

A checkpoint directory is recognised by its ``config.json`` (``architecture`` of the hybrid designs, else the Hugging Face
form that :mod:`kvmini.models.llama` reads); a preset name by the family that lists it."""

from __future__ import annotations

import glob
import json
import os
from typing import Any, Callable, Dict, Optional, Tuple

import torch

from . import gebasun, hybrid, llama, pipilix, vodinex, zipelix

# ``architecture`` in config.json -> its parser
ARCHITECTURES: Dict[str, Callable[..., Any]] = {m.ARCHITECTURE: m.config_from_json for m in (vodinex, pipilix, zipelix, gebasun)}
HYBRID_PRESETS: Dict[str, hybrid.HybridConfig] = {**vodinex.PRESETS, **pipilix.PRESETS, **zipelix.PRESETS, **gebasun.PRESETS}


def preset_names() -> Tuple[str, ...]:
    return tuple(llama.PRESETS) + tuple(HYBRID_PRESETS)


def resolve_model(model: str, weights_path: Optional[str] = None) -> "Tuple[Any, Optional[str]]":
    """(configuration, weights directory or None) of a preset name or a checkpoint directory."""
    path = os.path.join(model, "config.json")
    if os.path.isdir(model) and os.path.exists(path):
        with open(path) as f:
            arch = json.load(f).get("architecture")
        if arch is not None:
            if arch not in ARCHITECTURES:
                raise ValueError(f"{path}: architecture {arch!r} is not one this engine serves ({', '.join(ARCHITECTURES)})")
            if weights_path is None and glob.glob(os.path.join(model, "*.safetensors")):
                weights_path = model
            return ARCHITECTURES[arch](model), weights_path
    elif model.lower() in HYBRID_PRESETS:
        return HYBRID_PRESETS[model.lower()], weights_path
    return llama.resolve_model(model, weights_path)


def _hybrid_only(tp_size: int) -> None:
    if tp_size != 1:
        raise ValueError("tensor parallelism is not available for hybrid models")


def _pack_for(device: Any, dtype: torch.dtype, kernels: str) -> hybrid.Layout:
    """How matrices of a hybrid model are kept: fragment order for the bf16 kernels on a GPU, row-major otherwise."""
    if torch.device(device).type == "cuda" and kernels != "torch":
        from kvmini.ops.hip_mixers import layout

        return layout(dtype)
    return hybrid.Layout()


def load_weights(path: str, cfg: Any, device: Any = "cpu", dtype: torch.dtype = torch.bfloat16, tp_rank: int = 0, tp_size: int = 1, kernels: str = "auto") -> Any:
    """Weights from the ``*.safetensors`` of a directory (memory-mapped, a layer at a time)."""
    if not isinstance(cfg, hybrid.HybridConfig):
        return llama.load_hf_safetensors(path, cfg, device, dtype, tp_rank, tp_size)
    _hybrid_only(tp_size)
    from safetensors import safe_open

    files = sorted(glob.glob(os.path.join(path, "*.safetensors")))
    if not files:
        raise FileNotFoundError(f"no .safetensors files under {path}")
    where: Dict[str, Any] = {}
    for fpath in files:
        h = safe_open(fpath, framework="pt", device="cpu")
        where.update((k, h) for k in h.keys())

    def get(name: str) -> torch.Tensor:
        if name not in where:
            raise KeyError(f"{path}: tensor {name!r} is missing from the checkpoint")
        return where[name].get_tensor(name)

    return hybrid.build_weights(cfg, get, dtype, device, _pack_for(device, dtype, kernels))


def random_weights(cfg: Any, device: Any = "cpu", dtype: torch.dtype = torch.bfloat16, seed: int = 0, tp_rank: int = 0, tp_size: int = 1, tail_damping: Any = None,
                   kernels: str = "auto") -> Any:
    if not isinstance(cfg, hybrid.HybridConfig):
        return llama.random_weights(cfg, device, dtype, seed, tp_rank, tp_size, tail_damping=tail_damping)
    _hybrid_only(tp_size)
    return hybrid.build_weights(cfg, hybrid.random_tensors(cfg, device, dtype, seed), dtype, device, _pack_for(device, dtype, kernels))


def make_runner(weights: Any, rcfg: Any, tp_group: Any = None) -> Any:
    """The runner that executes these weights."""
    if isinstance(weights, hybrid.HybridWeights):
        from kvmini.engine.hybrid_runner import HybridRunner

        return HybridRunner(weights, rcfg, tp_group)
    from kvmini.engine.runner import ModelRunner

    return ModelRunner(weights, rcfg, tp_group)
