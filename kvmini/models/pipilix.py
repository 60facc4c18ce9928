"""Pipilix: a decoder of latent attention in sliding windows.  Every layer caches one normalised latent per token, from which
its heads' keys and values are linear maps; feed-forwards are silu-gated MLPs or mixtures of clamped experts; sublayers are
normalised on both sides; a stretch of layers runs several times with the same weights.  The configuration is the checkpoint's
own ``config.json``; tensors are named as :func:`kvmini.models.hybrid.tensor_shapes` lists them."""

from __future__ import annotations

import json
import os
from typing import Any, Dict, Optional, Tuple

from .hybrid import BranchSpec, HybridConfig, LatentSpec, LayerSpec, LoopSpec, MoeSpec

ARCHITECTURE = "Pipilix"


def _layer(i: int, la: Dict[str, Any]) -> LayerSpec:
    m, kind, mlp = la["mixer"], la["type"], la.get("mlp")
    if kind != "latent_attention":
        raise ValueError(f"layer {i}: unknown mixer {kind!r} (latent_attention)")
    size = int(m["mask"]["size"])
    if size < 1:
        raise ValueError(f"layer {i}: a window of {size} tokens")
    branches = (BranchSpec(LatentSpec(int(m["heads"]), int(m["dim"]), int(m["vdim"]), int(m["kv_rank"]), float(m["scale"]), size), "mix"),)
    if mlp is None:
        return LayerSpec(branches)
    if mlp.get("kind") == "dense":
        return LayerSpec(branches, int(mlp["ff"]), "silu")
    if mlp.get("kind") == "moe":
        r, e = mlp["router"], mlp["expert"]
        return LayerSpec(branches, moe=MoeSpec(int(r["experts"]), int(r["top"]), int(e["ff"]), float(e["limit"])))
    raise ValueError(f"layer {i}: unknown feed-forward {mlp.get('kind')!r} (dense, moe, or null for none)")


def config_from_json(doc: "str | Dict[str, Any]", name: Optional[str] = None) -> HybridConfig:
    if isinstance(doc, str):
        path = os.path.join(doc, "config.json") if os.path.isdir(doc) else doc
        with open(path) as f:
            d = json.load(f)
        name = name or os.path.basename(os.path.dirname(os.path.abspath(path)))
    else:
        d = doc
    if d.get("architecture") != ARCHITECTURE:
        raise ValueError(f"architecture {d.get('architecture')!r} is not {ARCHITECTURE}")
    lp = d.get("loop")
    return HybridConfig(name or "pipilix", int(d["vocab"]), int(d["width"]), tuple(_layer(i, la) for i, la in enumerate(d["layers"])), float(d["norm"]["eps"]), family="pipilix",
                        wiring="sandwich", embed_scale=float(d["embedding"]["scale"]), sine_positions=True, logit_scale=float(d["logit_scale"]),
                        loop=LoopSpec(int(lp["start"]), int(lp["stop"]), int(lp["times"])) if lp else None)


def stack(name: str, vocab: int, width: int, pattern: str, heads: int, dim: int, vdim: int, kv_rank: int, window: int, ff: int, experts: int, top: int, expert_ff: int,
          loop: Optional[Tuple[int, int, int]] = None, limit: float = 7.0, eps: float = 1e-6, embed_scale: float = 1.0, logit_scale: float = 1.0) -> HybridConfig:
    """A model of equal layers; ``pattern``: one letter a layer — D with an MLP, M with a mixture of experts, N without a feed-forward."""
    att = (BranchSpec(LatentSpec(heads, dim, vdim, kv_rank, dim ** -0.5, window), "mix"),)
    kinds = {"D": LayerSpec(att, ff, "silu"), "M": LayerSpec(att, moe=MoeSpec(experts, top, expert_ff, limit)), "N": LayerSpec(att)}
    return HybridConfig(name, vocab, width, tuple(kinds[c] for c in pattern), eps, family="pipilix", wiring="sandwich", embed_scale=embed_scale, sine_positions=True, logit_scale=logit_scale,
                        loop=LoopSpec(*loop) if loop else None)


PRESETS = {
    "pipilix-tiny": stack("pipilix-tiny", 512, 96, "DMN", 3, 24, 40, 48, 20, 112, 6, 2, 40, loop=(1, 3, 2), limit=2.0),
    # layers of the size of a 1B and an 8B decoder
    "pipilix-1b": stack("pipilix-1b", 128256, 2048, "D" + "M" * 11, 16, 128, 128, 512, 4096, 8192, 64, 6, 1408, loop=(4, 8, 2)),
    "pipilix-8b": stack("pipilix-8b", 128256, 4096, "D" + "M" * 23, 32, 128, 128, 512, 4096, 14336, 64, 6, 2304, loop=(8, 12, 2)),
}
