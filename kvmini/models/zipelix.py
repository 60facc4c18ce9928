"""Zipelix: a decoder whose layers mix tokens by latent attention or by retention, between several residual streams.  Latent
attention has a rotated key part beside the latent, a gate per output element, and may read the cache of an earlier layer;
retention is linear attention with a fixed decay per head.  Feed-forwards are silu-gated MLPs or mixtures of such experts with a
gated shared one; the LM head is the embedding table, logits are soft-capped.  The configuration is the checkpoint's own
``config.json``; tensors are named as :func:`kvmini.models.hybrid.tensor_shapes` lists them."""

from __future__ import annotations

import json
import os
from typing import Any, Dict, Optional, Tuple, Union

from .hybrid import BranchSpec, HybridConfig, LatentSpec, LayerSpec, MoeSpec, RetentionSpec

ARCHITECTURE = "Zipelix"


def _mixer(i: int, kind: str, m: Dict[str, Any]) -> Union[LatentSpec, RetentionSpec]:
    rot = m["rot"]
    if kind == "latent_attention":
        if int(rot["dims"]) != int(m["rot_dim"]):
            raise ValueError(f"layer {i}: {rot['dims']} of {m['rot_dim']} rotated dimensions turn (all of them do)")
        src = m.get("kv_from")
        return LatentSpec(int(m["heads"]), int(m["dim"]), int(m["vdim"]), int(m["kv_rank"]), float(m["scale"]), 0, int(m["rot_dim"]), float(rot["base"]), "element", -1 if src is None else int(src))
    if kind == "retention":
        return RetentionSpec(int(m["heads"]), int(m["dim"]), int(m["vdim"]), tuple(float(g) for g in m["decay"]), float(rot["base"]), int(rot["dims"]))
    raise ValueError(f"layer {i}: unknown mixer {kind!r} (latent_attention, retention)")


def _layer(i: int, la: Dict[str, Any]) -> LayerSpec:
    branches, mlp = (BranchSpec(_mixer(i, la["type"], la["mixer"]), "mix"),), la.get("mlp")
    if mlp is None:
        return LayerSpec(branches)
    if mlp.get("kind") == "dense":
        return LayerSpec(branches, int(mlp["ff"]), "silu")
    if mlp.get("kind") == "moe":
        r, sh = mlp["router"], mlp.get("shared")
        return LayerSpec(branches, moe=MoeSpec(int(r["experts"]), int(r["top"]), int(mlp["expert"]["ff"]), scores="softmax", scale=float(r["scale"]), correction=False, act="silu",
                                               shared_ff=int(sh["ff"]) if sh else 0))
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
    return HybridConfig(name or "zipelix", int(d["vocab"]), int(d["width"]), tuple(_layer(i, la) for i, la in enumerate(d["layers"])), float(d["norm"]["eps"]), family="zipelix", wiring="hyper",
                        streams=int(d["streams"]), tied_head=True, logit_softcap=float(d["logit_softcap"]))


def stack(name: str, vocab: int, width: int, pattern: str, heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, ret_heads: int, ret_dim: int, ret_vdim: int, ff: int, experts: int, top: int,
          expert_ff: int, shared_ff: int, streams: int = 2, router_scale: float = 1.0, rot_base: float = 500000.0, softcap: float = 30.0, eps: float = 1e-6) -> HybridConfig:
    """A model of equal layers; ``pattern``: two letters a layer — L latent attention, S the same on the last L layer's cache, R
    retention; then D with an MLP, M with a mixture of experts, N without a feed-forward."""
    ff_kinds: Dict[str, Dict[str, Any]] = {"D": dict(ff=ff, act="silu"), "N": {},
                                           "M": dict(moe=MoeSpec(experts, top, expert_ff, scores="softmax", scale=router_scale, correction=False, act="silu", shared_ff=shared_ff))}
    decay = tuple(1.0 - 2.0 ** (-5.0 - 7.0 * h / max(1, ret_heads)) for h in range(ret_heads))
    layers, last = [], -1
    for i, (kind, mlp) in enumerate(zip(pattern[::2], pattern[1::2])):
        if kind == "L":
            last = i
        m = RetentionSpec(ret_heads, ret_dim, ret_vdim, decay, rot_base, ret_dim) if kind == "R" else \
            LatentSpec(heads, dim, vdim, kv_rank, (dim + rot_dim) ** -0.5, 0, rot_dim, rot_base, "element", last if kind == "S" else -1)
        layers.append(LayerSpec((BranchSpec(m, "mix"),), **ff_kinds[mlp]))
    return HybridConfig(name, vocab, width, tuple(layers), eps, family="zipelix", wiring="hyper", streams=streams, tied_head=True, logit_softcap=softcap)


PRESETS = {
    "zipelix-tiny": stack("zipelix-tiny", 512, 96, "LDRMSMRNSD", 3, 24, 8, 40, 48, 2, 24, 20, 112, 6, 2, 40, 56, streams=3),
    # layers of the size of a 1B and an 8B decoder
    "zipelix-1b": stack("zipelix-1b", 128256, 2048, "LDRMSMRM" * 3, 16, 128, 64, 128, 512, 16, 128, 128, 8192, 64, 6, 1408, 2816),
    "zipelix-8b": stack("zipelix-8b", 128256, 4096, "LDRMSMRM" * 6, 32, 128, 64, 128, 512, 32, 128, 128, 14336, 64, 6, 2304, 4608),
}
