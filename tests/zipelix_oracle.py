"""Plain, slow model of the Zipelix design for the tests: one function per mechanism, a sequence at a time, no cache, no
batching, nothing shared with the engine.  Works in whatever floating type the weights are given in (the tests use
float64), reads a configuration as the parsed ``config.json`` and the weights as a dict of tensors."""

from __future__ import annotations

import math
from typing import Any, Dict, List, Optional, Tuple

import torch

Weights = Dict[str, torch.Tensor]
Margins = Optional[List[torch.Tensor]]


def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x over its root mean square along the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z / (1 + torch.exp(-z))


def _angles(n: int, dims: int, base: float, first: int) -> torch.Tensor:
    freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    return torch.arange(first, first + n, dtype=torch.float64)[:, None] * freq


def rotate_neighbours(x: torch.Tensor, dims: int, base: float, first: int = 0) -> torch.Tensor:
    """x [T, heads, n]: entries 2 i and 2 i + 1 of the first ``dims`` turn together."""
    out = x.clone()
    a = _angles(x.shape[0], dims, base, first).to(x.dtype)
    for i in range(dims // 2):
        c, s = torch.cos(a[:, i])[:, None], torch.sin(a[:, i])[:, None]
        out[..., 2 * i] = x[..., 2 * i] * c - x[..., 2 * i + 1] * s
        out[..., 2 * i + 1] = x[..., 2 * i + 1] * c + x[..., 2 * i] * s
    return out


def rotate_halves(x: torch.Tensor, dims: int, base: float, first: int = 0) -> torch.Tensor:
    """x [T, heads, n]: entries i and i + dims / 2 of the first ``dims`` turn together."""
    out = x.clone()
    a = _angles(x.shape[0], dims, base, first).to(x.dtype)
    for i in range(dims // 2):
        j = i + dims // 2
        c, s = torch.cos(a[:, i])[:, None], torch.sin(a[:, i])[:, None]
        out[..., i] = x[..., i] * c - x[..., j] * s
        out[..., j] = x[..., j] * c + x[..., i] * s
    return out


def causal_softmax_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float) -> torch.Tensor:
    """q, k [T, H, dim], v [T, H, vdim] -> [T, H, vdim]; every head has its own keys and values."""
    t, nh = q.shape[:2]
    out = torch.zeros(t, nh, v.shape[2], dtype=q.dtype)
    for i in range(t):
        s = torch.einsum("hd,jhd->hj", q[i], k[: i + 1]) * scale
        p = torch.exp(s - s.max(-1, keepdim=True).values)
        out[i] = torch.einsum("hj,jhd->hd", p / p.sum(-1, keepdim=True), v[: i + 1])
    return out


def latents(h: torch.Tensor, w: Weights, name: str, m: Dict[str, Any], eps: float) -> Tuple[torch.Tensor, torch.Tensor]:
    """(normed latent [T, kv_rank], rotated key part [T, rot_dim]) that a layer with a latent of its own makes."""
    z, r = h @ w[name + ".dkv"].T, m["kv_rank"]
    return rms_unit(z[:, :r], eps) * w[name + ".dkv.norm"], rotate_neighbours(z[:, None, r:], m["rot_dim"], m["rot"]["base"])[:, 0]


def latent_attention(h: torch.Tensor, w: Weights, name: str, m: Dict[str, Any], kv: Tuple[torch.Tensor, torch.Tensor]) -> torch.Tensor:
    t, nh, d, dr, dv = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, kr = kv
    q = (h @ w[name + ".q"].T).view(t, nh, d + dr)
    q = torch.cat((q[..., :d], rotate_neighbours(q[..., d:], dr, m["rot"]["base"])), -1)
    k = torch.cat(((c @ w[name + ".uk"].T).view(t, nh, d), kr[:, None].expand(t, nh, dr)), -1)
    v = (c @ w[name + ".uv"].T).view(t, nh, dv)
    a = causal_softmax_attention(q, k, v, m["scale"]).reshape(t, nh * dv)
    return (a * torch.sigmoid(h @ w[name + ".g"].T)) @ w[name + ".o"].T


def decaying_sums(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: List[float]) -> torch.Tensor:
    """Token by token: S <- decay S + k v^T, o = S^T q.  q, k [T, H, dim], v [T, H, vdim]."""
    t, nh, d = q.shape
    g = torch.tensor(decay, dtype=q.dtype)[:, None, None]
    s, out = torch.zeros(nh, d, v.shape[2], dtype=q.dtype), []
    for i in range(t):
        s = g * s + k[i][:, :, None] * v[i][:, None, :]
        out.append((s * q[i][:, :, None]).sum(1))
    return torch.stack(out)


def retention(h: torch.Tensor, w: Weights, name: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    t, nh, d, dv, rot = h.shape[0], m["heads"], m["dim"], m["vdim"], m["rot"]
    q = rotate_halves((h @ w[name + ".q"].T).view(t, nh, d), rot["dims"], rot["base"])
    k = rotate_halves((h @ w[name + ".k"].T).view(t, nh, d), rot["dims"], rot["base"]) / math.sqrt(d)
    o = rms_unit(decaying_sums(q, k, (h @ w[name + ".v"].T).view(t, nh, dv), m["decay"]), eps).reshape(t, nh * dv)
    return (o * silu(h @ w[name + ".g"].T)) @ w[name + ".o"].T


def gated_mlp(h: torch.Tensor, w: Weights, name: str) -> torch.Tensor:
    return (silu(h @ w[name + ".gate"].T) * (h @ w[name + ".up"].T)) @ w[name + ".down"].T


def choose_experts(z: torch.Tensor, top: int, scale: float) -> Tuple[torch.Tensor, torch.Tensor]:
    """Router logits [T, E] -> (experts [T, top], their weights: shares of the softmax over all, times scale)."""
    s = torch.exp(z - z.max(-1, keepdim=True).values)
    s = s / s.sum(-1, keepdim=True)
    idx = torch.topk(s, top, dim=-1).indices
    return idx, s.gather(-1, idx) * scale


def choice_margin(z: torch.Tensor, top: int) -> torch.Tensor:
    """By how much (in logits) the last chosen expert beat the first one left out, [T]."""
    c = z.sort(-1, descending=True).values
    return c[:, top - 1] - c[:, top] if top < z.shape[1] else torch.full((z.shape[0],), float("inf"), dtype=z.dtype)


def mixture(h: torch.Tensor, w: Weights, name: str, m: Dict[str, Any], margins: Margins = None) -> torch.Tensor:
    z = h @ w[name + ".router"].T
    idx, wt = choose_experts(z, m["router"]["top"], m["router"]["scale"])
    if margins is not None:
        margins.append(choice_margin(z, m["router"]["top"]))
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(idx[t].tolist(), wt[t]):
            out[t] += s * gated_mlp(h[t : t + 1], w, f"{name}.e{e}")[0]
    if m.get("shared"):
        out = out + torch.sigmoid(h @ w[name + ".shared.sg"].T) * gated_mlp(h, w, name + ".shared")
    return out


def read_streams(x: torch.Tensor, w: Weights, name: str) -> torch.Tensor:
    """x [streams, T, width] -> the sublayer's input."""
    return sum(w[name + ".in"][s] * x[s] for s in range(x.shape[0]))


def write_streams(x: torch.Tensor, y: torch.Tensor, w: Weights, name: str) -> torch.Tensor:
    """Every stream anew from all old ones (mix [from, to]) and the sublayer's result."""
    n, mix, out = x.shape[0], w[name + ".mix"], w[name + ".out"]
    return torch.stack([sum(mix[s, t] * x[s] for s in range(n)) + out[t] * y for t in range(n)])


def layer_outputs(doc: Dict[str, Any], w: Weights, toks: List[int], margins: Margins = None) -> List[torch.Tensor]:
    """The sum of the streams behind every layer."""
    eps, out = doc["norm"]["eps"], []
    x = w["embed"][toks][None].repeat(doc["streams"], 1, 1)
    made: Dict[int, Tuple[torch.Tensor, torch.Tensor]] = {}
    for i, la in enumerate(doc["layers"]):
        n, m = f"l{i}", la["mixer"]
        h = rms_unit(read_streams(x, w, n + ".hc1"), eps) * w[n + ".norm1"]
        if la["type"] == "retention":
            y = retention(h, w, n + ".mix", m, eps)
        else:
            if "kv_from" not in m:
                made[i] = latents(h, w, n + ".mix", m, eps)
            y = latent_attention(h, w, n + ".mix", m, made[m.get("kv_from", i)])
        x = write_streams(x, y, w, n + ".hc1")
        mlp = la["mlp"]
        if mlp is not None:
            h = rms_unit(read_streams(x, w, n + ".hc2"), eps) * w[n + ".norm2"]
            y = gated_mlp(h, w, n + ".mlp") if mlp["kind"] == "dense" else mixture(h, w, n + ".mlp", mlp, margins)
            x = write_streams(x, y, w, n + ".hc2")
        out.append(x.sum(0))
    return out


def closest_choices(doc: Dict[str, Any], w: Weights, toks: List[int]) -> torch.Tensor:
    """Per position, the smallest margin of any of its choices of experts."""
    margins: List[torch.Tensor] = [torch.full((len(toks),), float("inf"), dtype=torch.float64)]
    layer_outputs(doc, w, toks, margins)
    return torch.stack([m.double() for m in margins]).min(0).values


def capped(z: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(z / cap)


def logits(doc: Dict[str, Any], w: Weights, toks: List[int]) -> torch.Tensor:
    x = layer_outputs(doc, w, toks)[-1]
    return capped((rms_unit(x, doc["norm"]["eps"]) * w["final.norm"]) @ w["embed"].T, doc["logit_softcap"])


def greedy(doc: Dict[str, Any], w: Weights, prompt: List[int], n: int) -> List[int]:
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(logits(doc, w, toks)[-1].argmax()))
    return toks[len(prompt) :]
