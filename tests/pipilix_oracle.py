"""Plain, slow model of the Pipilix design for the tests: one function per mechanism, a sequence at a time, no cache, no
batching, nothing shared with the engine.  Works in whatever floating type the weights are given in (the tests use
float64), reads a configuration as the parsed ``config.json`` and the weights as a dict of tensors."""

from __future__ import annotations

from typing import Any, Dict, List, Optional, Tuple

import torch

Weights = Dict[str, torch.Tensor]
Margins = Optional[List[torch.Tensor]]


def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x over its root mean square along the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sine_positions(n: int, width: int, first: int = 0) -> torch.Tensor:
    """[n, width]: sine in even entries, cosine in odd ones, of position times 10000^(-2 (entry // 2) / width)."""
    out = torch.zeros(n, width, dtype=torch.float64)
    for e in range(width):
        a = torch.arange(first, first + n, dtype=torch.float64) * 10000.0 ** (-2.0 * (e // 2) / width)
        out[:, e] = torch.cos(a) if e % 2 else torch.sin(a)
    return out


def embedding(toks: List[int], w: Weights, scale: float) -> torch.Tensor:
    x = w["embed"][toks] * scale
    return x + sine_positions(len(toks), x.shape[1]).to(x.dtype)


def visible_in_window(i: int, j: int, size: int) -> bool:
    return 0 <= i - j < size


def windowed_softmax_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, size: int) -> torch.Tensor:
    """q, k [T, H, dim], v [T, H, vdim] -> [T, H, vdim]; every head has its own keys and values."""
    t, nh = q.shape[:2]
    out = torch.zeros(t, nh, v.shape[2], dtype=q.dtype)
    for i in range(t):
        first = max(0, i - size + 1)
        for h in range(nh):
            s = (k[first : i + 1, h] @ q[i, h]) * scale
            p = torch.exp(s - s.max())
            out[i, h] = (p / p.sum()) @ v[first : i + 1, h]
    return out


def latent_attention(h: torch.Tensor, w: Weights, name: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    t, nh, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[name + ".q"].T).view(t, nh, d)
    c = rms_unit(h @ w[name + ".dkv"].T, eps) * w[name + ".dkv.norm"]
    k = (c @ w[name + ".uk"].T).view(t, nh, d)
    v = (c @ w[name + ".uv"].T).view(t, nh, dv)
    a = windowed_softmax_attention(q, k, v, m["scale"], m["mask"]["size"])
    a = a * torch.sigmoid(h @ w[name + ".g"].T)[:, :, None]
    return a.reshape(t, nh * dv) @ w[name + ".o"].T


def silu_gated_mlp(h: torch.Tensor, w: Weights, name: str) -> torch.Tensor:
    z = h @ w[name + ".gate"].T
    return (z * torch.sigmoid(z) * (h @ w[name + ".up"].T)) @ w[name + ".down"].T


def clamped_gate(gate: torch.Tensor, up: torch.Tensor, limit: float) -> torch.Tensor:
    g, u = gate.clamp(max=limit), up.clamp(-limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


def expert(h: torch.Tensor, w: Weights, name: str, limit: float) -> torch.Tensor:
    return clamped_gate(h @ w[name + ".gate"].T, h @ w[name + ".up"].T, limit) @ w[name + ".down"].T


def choose_experts(z: torch.Tensor, correction: torch.Tensor, top: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """Router logits [T, E] -> (experts [T, top] by corrected score, their weights: the scores themselves)."""
    s = torch.sigmoid(z)
    idx = torch.topk(s + correction, top, dim=-1).indices
    return idx, s.gather(-1, idx)


def choice_margin(z: torch.Tensor, correction: torch.Tensor, top: int) -> torch.Tensor:
    """By how much the last chosen expert beat the first one left out, [T]."""
    c = (torch.sigmoid(z) + correction).sort(-1, descending=True).values
    return c[:, top - 1] - c[:, top] if top < z.shape[1] else torch.full((z.shape[0],), float("inf"), dtype=z.dtype)


def mixture(h: torch.Tensor, w: Weights, name: str, m: Dict[str, Any], margins: Margins = None) -> torch.Tensor:
    z = h @ w[name + ".router"].T
    idx, wt = choose_experts(z, w[name + ".correction"], m["router"]["top"])
    if margins is not None:
        margins.append(choice_margin(z, w[name + ".correction"], m["router"]["top"]))
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(idx[t].tolist(), wt[t]):
            out[t] += s * expert(h[t : t + 1], w, f"{name}.e{e}", m["expert"]["limit"])[0]
    return out


def layer(x: torch.Tensor, w: Weights, name: str, la: Dict[str, Any], eps: float, margins: Margins = None) -> torch.Tensor:
    def norm(v: torch.Tensor, n: str) -> torch.Tensor:
        return rms_unit(v, eps) * w[f"{name}.{n}"]

    x = x + norm(latent_attention(norm(x, "norm1"), w, name + ".mix", la["mixer"], eps), "norm1b")
    m = la["mlp"]
    if m is not None:
        h = norm(x, "norm2")
        x = x + norm(silu_gated_mlp(h, w, name + ".mlp") if m["kind"] == "dense" else mixture(h, w, name + ".mlp", m, margins), "norm2b")
    return x


def layer_order(doc: Dict[str, Any]) -> List[Tuple[int, Optional[int]]]:
    """(layer, pass that begins right before it or None) in the order they run."""
    lp = doc.get("loop") or {"start": 0, "stop": 0, "times": 0}
    out: List[Tuple[int, Optional[int]]] = [(i, None) for i in range(lp["start"])]
    for t in range(lp["times"]):
        out += [(i, t if i == lp["start"] else None) for i in range(lp["start"], lp["stop"])]
    return out + [(i, None) for i in range(lp["stop"], len(doc["layers"]))]


def layer_outputs(doc: Dict[str, Any], w: Weights, toks: List[int], margins: Margins = None) -> List[torch.Tensor]:
    """The residual stream behind every layer run."""
    e = embedding(toks, w, doc["embedding"]["scale"])
    x, out = e, []
    for i, begins in layer_order(doc):
        if begins is not None:
            if begins > 0:
                x = x + e
            x = x + w["loop.step"][begins]
        x = layer(x, w, f"l{i}", doc["layers"][i], doc["norm"]["eps"], margins)
        out.append(x)
    return out


def closest_choices(doc: Dict[str, Any], w: Weights, toks: List[int]) -> torch.Tensor:
    """Per position, the smallest margin of any of its choices of experts."""
    margins: List[torch.Tensor] = [torch.full((len(toks),), float("inf"), dtype=torch.float64)]
    layer_outputs(doc, w, toks, margins)
    return torch.stack([m.double() for m in margins]).min(0).values


def logits(doc: Dict[str, Any], w: Weights, toks: List[int]) -> torch.Tensor:
    x = layer_outputs(doc, w, toks)[-1]
    return (rms_unit(x, doc["norm"]["eps"]) * w["final.norm"]) @ w["head"].T * doc["logit_scale"]


def greedy(doc: Dict[str, Any], w: Weights, prompt: List[int], n: int) -> List[int]:
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(logits(doc, w, toks)[-1].argmax()))
    return toks[len(prompt) :]
