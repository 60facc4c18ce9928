"""Gebasun: a decoder whose layers mix tokens by one of two kinds of sliding-window attention or by a selective state space.  Both
kinds of attention take the keys, as projected, for their values, norm queries and keys without gains and have a sink per head; one
(``attention``) tells positions by a learned bias per distance, the other (``attention_2``) rotates part of a head, keeps the first
tokens of the sequence in sight and gates its output element by element.  Feed-forwards are mixtures of squared-relu experts beside a
shared one, chosen by the router's logits and weighted by the softmax over the chosen; mixer and feed-forward of a layer read the same
stream, each behind its own norm.  The configuration is the checkpoint's own ``config.json``; tensors are named as
:func:`kvmini.models.hybrid.tensor_shapes` lists them."""

from __future__ import annotations

import json
import os
from typing import Any, Dict, Optional, Union

from .hybrid import AttentionSpec, BranchSpec, HybridConfig, LayerSpec, MoeSpec, StateSpaceSpec

ARCHITECTURE = "Gebasun"


def _mixer(i: int, kind: str, m: Dict[str, Any]) -> Union[AttentionSpec, StateSpaceSpec]:
    if kind == "mamba2":
        return StateSpaceSpec(int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"]), int(m["conv"]), int(m["norm_groups"]))
    if kind not in ("attention", "attention_2"):
        raise ValueError(f"layer {i}: unknown mixer {kind!r} (attention, attention_2, mamba2)")
    size = int(m["mask"]["size"])
    if size < 1:
        raise ValueError(f"layer {i}: a window of {size} tokens")
    heads = (int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), float(m["scale"]))
    if kind == "attention":
        return AttentionSpec(*heads, window=size, gate="none", key_values=True, norm_gains=False, sink=True, rel=True, rel_max=int(m["bias_max"]))
    return AttentionSpec(*heads, 0, float(m["rot"]["base"]), int(m["rot"]["dims"]), size, int(m["mask"]["keep_first"]), "element", True, False, out_bias=False, sink=True)


def _layer(i: int, la: Dict[str, Any]) -> LayerSpec:
    branches, mlp = (BranchSpec(_mixer(i, la["type"], la["mixer"]), "mix"),), la.get("mlp")
    if mlp is None:
        return LayerSpec(branches)
    if mlp.get("kind") != "moe":
        raise ValueError(f"layer {i}: unknown feed-forward {mlp.get('kind')!r} (moe, or null for none)")
    r, sh = mlp["router"], mlp.get("shared")
    return LayerSpec(branches, moe=_experts(int(r["experts"]), int(r["top"]), int(mlp["expert"]["ff"]), int(sh["ff"]) if sh else 0))


def _experts(experts: int, top: int, ff: int, shared_ff: int) -> MoeSpec:
    return MoeSpec(experts, top, ff, scores="chosen", correction=False, act="relu2", shared_ff=shared_ff, shared_gate=False, bias=True)


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
    return HybridConfig(name or "gebasun", int(d["vocab"]), int(d["width"]), tuple(_layer(i, la) for i, la in enumerate(d["layers"])), float(d["norm"]["eps"]), family="gebasun", wiring="parallel")


def stack(name: str, vocab: int, width: int, pattern: str, heads: int, kv_heads: int, dim: int, window: int, keep: int, rot_dims: int, ssm_heads: int, ssm_vdim: int, ssm_state: int, ssm_groups: int,
          experts: int, top: int, expert_ff: int, shared_ff: int, taps: int = 4, norm_groups: int = 1, buckets: int = 32, rel_max: int = 1024, base: float = 500000.0, scale: Optional[float] = None,
          eps: float = 1e-6) -> HybridConfig:
    """A model of equal layers; ``pattern``: two letters a layer — A attention with a distance bias, B rotated attention that keeps the first
    tokens, S state space; then M with a mixture of experts, N without a feed-forward."""
    common: Dict[str, Any] = dict(key_values=True, norm_gains=False, sink=True)
    sizes = (heads, kv_heads, dim, dim, dim ** -0.5 if scale is None else scale)
    mixers: Dict[str, Union[AttentionSpec, StateSpaceSpec]] = {
        "A": AttentionSpec(*sizes, window=window, gate="none", rel=True, rel_max=rel_max, rel_buckets=buckets, **common),
        "B": AttentionSpec(*sizes, 0, base, rot_dims, window, keep, "element", out_bias=False, **common),
        "S": StateSpaceSpec(ssm_heads, ssm_vdim, ssm_state, ssm_groups, taps, norm_groups)}
    moe = {"M": _experts(experts, top, expert_ff, shared_ff), "N": None}
    layers = tuple(LayerSpec((BranchSpec(mixers[a], "mix"),), moe=moe[f]) for a, f in zip(pattern[::2], pattern[1::2]))
    return HybridConfig(name, vocab, width, layers, eps, family="gebasun", wiring="parallel")


PRESETS = {
    "gebasun-tiny": stack("gebasun-tiny", 512, 96, "BMSMAMSNBM", 4, 2, 24, 40, 3, 10, 3, 20, 24, 1, 6, 2, 40, 56, rel_max=30, buckets=12),
    # layers of the size of a 1B and an 8B decoder
    "gebasun-1b": stack("gebasun-1b", 128256, 2048, "BMSMAMSM" * 3, 16, 4, 128, 4096, 64, 64, 64, 64, 128, 1, 64, 6, 1408, 2816),
    "gebasun-8b": stack("gebasun-8b", 128256, 4096, "BMSMAMSM" * 6, 32, 8, 128, 4096, 64, 64, 128, 64, 128, 1, 64, 6, 2304, 4608),
}
