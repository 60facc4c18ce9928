"""Plain, slow model of the Gebasun design for the tests: one function per mechanism, a sequence at a time, no cache, no
batching, nothing shared with the engine.  Works in whatever floating type the weights are given in (the tests use
float64), reads a configuration as the parsed ``config.json`` and the weights as a dict of tensors."""

from __future__ import annotations

import math
from typing import Any, Callable, Dict, List, Optional, Tuple

import torch

Weights = Dict[str, torch.Tensor]
Margins = Optional[List[torch.Tensor]]


def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x over its root mean square along the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z / (1 + torch.exp(-z))


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def rotate_halves(x: torch.Tensor, dims: int, base: float, first: int = 0) -> torch.Tensor:
    """x [T, heads, n]: entries i and i + dims / 2 of the first ``dims`` turn together."""
    out = x.clone()
    for i in range(dims // 2):
        a = (torch.arange(first, first + x.shape[0], dtype=torch.float64) * base ** (-2.0 * i / dims)).to(x.dtype)
        c, s, j = torch.cos(a)[:, None], torch.sin(a)[:, None], i + dims // 2
        out[..., i] = x[..., i] * c - x[..., j] * s
        out[..., j] = x[..., j] * c + x[..., i] * s
    return out


def distance_bucket(n: int, buckets: int, longest: int) -> int:
    """Row of the bias table for a key ``n`` tokens back: one each for short distances, then logarithmically wider ones."""
    half = buckets / 2
    if n < half:
        return n
    return min(buckets - 1, int(half + math.floor(math.log(n / half) / math.log(longest / half) * (buckets - half))))


def sees(i: int, j: int, window: int, keep: int = 0) -> bool:
    return j <= i and (i - j < window or j < keep)


def softmax_with_sink(s: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """s [heads, keys], sink [heads]: the weights of the keys; the sink takes its share and gives nothing."""
    top = torch.maximum(s.max(-1).values, sink)[:, None]
    p = torch.exp(s - top)
    return p / (p.sum(-1, keepdim=True) + torch.exp(sink[:, None] - top))


def attend(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, sink: torch.Tensor, visible: Callable[[int, int], bool],
           bias: Optional[Callable[[int], torch.Tensor]] = None) -> torch.Tensor:
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H, vdim]; ``bias(n)``: [H], added to the scores of keys n back."""
    t, nh = q.shape[:2]
    group = [h // (nh // k.shape[1]) for h in range(nh)]
    out = torch.zeros(t, nh, v.shape[2], dtype=q.dtype)
    for i in range(t):
        js = [j for j in range(i + 1) if visible(i, j)]
        s = torch.einsum("hd,jhd->hj", q[i], k[js][:, group]) * scale
        if bias is not None:
            s = s + torch.stack([bias(i - j) for j in js], 1)
        out[i] = torch.einsum("hj,jhd->hd", softmax_with_sink(s, sink), v[js][:, group])
    return out


def attention(h: torch.Tensor, w: Weights, name: str, kind: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    t, nh, g, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = (h @ w[name + ".q"].T + w[name + ".q.b"]).view(t, nh, d)
    k = (h @ w[name + ".k"].T + w[name + ".k.b"]).view(t, g, d)
    v, bias = k, None
    if kind == "attention_2":
        q, k = (rotate_halves(x, m["rot"]["dims"], m["rot"]["base"]) for x in (q, k))
    else:
        rel = w[name + ".rel"]
        bias = lambda n: rel[distance_bucket(n, rel.shape[0], m["bias_max"])]  # noqa: E731
    window, keep = m["mask"]["size"], m["mask"].get("keep_first", 0)
    o = attend(rms_unit(q, eps), rms_unit(k, eps), v, m["scale"], w[name + ".sink"], lambda i, j: sees(i, j, window, keep), bias).reshape(t, nh * d)
    if kind == "attention_2":
        return (o / (1 + torch.exp(-(h @ w[name + ".g"].T)))) @ w[name + ".o"].T
    return o @ w[name + ".o"].T + w[name + ".o.b"]


def causal_convolution(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """x [T, channels], taps [channels, n] (the last one is the current token's)."""
    n = taps.shape[1]
    ext = torch.cat((torch.zeros(n - 1, x.shape[1], dtype=x.dtype), x))
    return sum(ext[j : j + x.shape[0]] * taps[:, j] for j in range(n)) + bias


def selective_sums(x: torch.Tensor, b: torch.Tensor, c: torch.Tensor, dt: torch.Tensor, a_log: torch.Tensor, d: torch.Tensor) -> torch.Tensor:
    """Token by token: S <- exp(-exp(A) dt) S + dt b x^T, y = S^T c + D x.  x [T, H, P], b and c [T, G, N], dt [T, H]."""
    t, nh, p = x.shape
    g, n = b.shape[1:]
    group = [h // (nh // g) for h in range(nh)]
    s, out = torch.zeros(nh, n, p, dtype=x.dtype), []
    for i in range(t):
        s = torch.exp(-torch.exp(a_log) * dt[i])[:, None, None] * s + dt[i][:, None, None] * b[i][group][:, :, None] * x[i][:, None, :]
        out.append((s * c[i][group][:, :, None]).sum(1) + d[:, None] * x[i])
    return torch.stack(out)


def gated_group_norm(y: torch.Tensor, z: torch.Tensor, parts: int, gain: torch.Tensor, eps: float) -> torch.Tensor:
    """y times silu(z), then each of ``parts`` equal parts over its own root mean square, times the gain."""
    r = y * silu(z)
    return rms_unit(r.view(r.shape[0], parts, -1), eps).reshape(r.shape) * gain


def mamba2(h: torch.Tensor, w: Weights, name: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    t, nh, p, g, n = h.shape[0], m["heads"], m["vdim"], m["groups"], m["state"]
    z, xbc, dt = (h @ w[name + ".in"].T).split([nh * p, nh * p + 2 * g * n, nh], -1)
    xbc = silu(causal_convolution(xbc, w[name + ".conv"], w[name + ".conv.b"]))
    x, b, c = xbc.split([nh * p, g * n, g * n], -1)
    y = selective_sums(x.view(t, nh, p), b.view(t, g, n), c.view(t, g, n), softplus(dt + w[name + ".dt_bias"]), w[name + ".A_log"], w[name + ".D"])
    return gated_group_norm(y.reshape(t, nh * p), z, m["norm_groups"], w[name + ".norm"], eps) @ w[name + ".o"].T


def expert(h: torch.Tensor, w: Weights, name: str) -> torch.Tensor:
    return torch.clamp(h @ w[name + ".up"].T, min=0) ** 2 @ w[name + ".down"].T


def choose_experts(z: torch.Tensor, top: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """Router logits [T, E] -> (experts [T, top], their weights: the softmax over the chosen logits alone)."""
    v, idx = torch.topk(z, top, dim=-1)
    e = torch.exp(v - v[:, :1])
    return idx, e / e.sum(-1, keepdim=True)


def choice_margin(z: torch.Tensor, top: int) -> torch.Tensor:
    """By how much the last chosen expert beat the first one left out, [T]."""
    c = z.sort(-1, descending=True).values
    return c[:, top - 1] - c[:, top] if top < z.shape[1] else torch.full((z.shape[0],), float("inf"), dtype=z.dtype)


def mixture(h: torch.Tensor, w: Weights, name: str, m: Dict[str, Any], margins: Margins = None) -> torch.Tensor:
    z = h @ w[name + ".router"].T + w[name + ".router.b"]
    idx, wt = choose_experts(z, m["router"]["top"])
    if margins is not None:
        margins.append(choice_margin(z, m["router"]["top"]))
    out = expert(h, w, name + ".shared") if m.get("shared") else torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        t, k = (idx == e).nonzero(as_tuple=True)
        if len(t):
            out[t] = out[t] + wt[t, k][:, None] * expert(h[t], w, f"{name}.e{e}")
    return out


def layer_outputs(doc: Dict[str, Any], w: Weights, toks: List[int], margins: Margins = None) -> List[torch.Tensor]:
    """The residual stream behind every layer."""
    eps, out = doc["norm"]["eps"], []
    x = w["embed"][toks]
    for i, la in enumerate(doc["layers"]):
        n, kind, m, mlp = f"l{i}", la["type"], la["mixer"], la["mlp"]
        h = rms_unit(x, eps) * w[n + ".norm1"]
        y = mamba2(h, w, n + ".mix", m, eps) if kind == "mamba2" else attention(h, w, n + ".mix", kind, m, eps)
        if mlp is not None:
            y = y + mixture(rms_unit(x, eps) * w[n + ".norm2"], w, n + ".mlp", mlp, margins)
        x = x + y
        out.append(x)
    return out


def closest_choices(doc: Dict[str, Any], w: Weights, toks: List[int]) -> torch.Tensor:
    """Per position, the smallest margin of any of its choices of experts."""
    margins: List[torch.Tensor] = [torch.full((len(toks),), float("inf"), dtype=torch.float64)]
    layer_outputs(doc, w, toks, margins)
    return torch.stack([m.double() for m in margins]).min(0).values


def logits(doc: Dict[str, Any], w: Weights, toks: List[int]) -> torch.Tensor:
    x = layer_outputs(doc, w, toks)[-1]
    return (rms_unit(x, doc["norm"]["eps"]) * w["final.norm"]) @ w["head"].T


def greedy(doc: Dict[str, Any], w: Weights, prompt: List[int], n: int) -> List[int]:
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(logits(doc, w, toks)[-1].argmax()))
    return toks[len(prompt) :]
