"""Plain-PyTorch sequence mixers (CPU execution; the HIP form is :mod:`kvmini.ops.hip_mixers`, same call surface).

A step's tokens are rows of flat ``[T, ...]`` tensors, portions of several sequences one after the other.  :class:`Step`
carries what the runner staged about them.  The residual stream, norms, gates, scores and the recurrence are fp32 whatever
the activations' type."""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Tuple

import torch
import torch.nn.functional as F

from kvmini.models.hybrid import AttentionSpec, AttentionWeights, DeltaSpec, DeltaWeights, HyperWeights, LatentSpec, LatentWeights, MoeSpec, MoeWeights, RetentionSpec, RetentionWeights, \
    StateSpaceSpec, StateSpaceWeights


@dataclass
class Step:
    tokens: torch.Tensor  # [T] int32, as the following per-token arrays
    positions: torch.Tensor
    slots: torch.Tensor  # cache slot of the token's K / V (block * block_size + offset; -1: padding row)
    tok_seq: torch.Tensor  # sequence slot: row of block_tables and of the recurrent state
    tok_kind: torch.Tensor  # 0 padding, 1 the only token of its sequence in this step, 2 a token of a longer portion
    tok_off: torch.Tensor  # index of the token inside its portion
    block_tables: torch.Tensor  # [sequences, blocks]
    singles: torch.Tensor  # rows that are the only token of their sequence in this step (-1 = unused)
    portions: torch.Tensor  # [5, n]: first row, tokens (0 = unused), first position, sequence slot, first tile
    blocks: torch.Tensor  # [4, m]: query blocks of at most 32 tokens of portions of several tokens: first row, tokens (0 = unused), first position, sequence slot
    n_blocks: int  # at most that many of them are in use
    tiles: torch.Tensor  # [4, k]: the same in tiles of 16, at most the first n_tiles of them in use
    n_tiles: int
    decode_only: bool  # every row is padding or the only token of its sequence
    long: bool = False  # decode_only, with a context long enough to be shared out over several workgroups
    # prompts of latent attention, for ops that expand keys and values into a workspace:
    spans: Optional[torch.Tensor] = None  # [3, sequences]: first workspace row, first position, rows (0 = none) of a sequence's portion and what its windows reach
    span_rows: int = 0  # rows of the workspace
    latent_blocks: Optional[torch.Tensor] = None  # [4, m]: query blocks of at most 128 tokens: first row, tokens (0 = unused), first position, workspace row of position 0
    n_latent_blocks: int = 0  # at most that many of them are in use
    gathered: Dict[int, torch.Tensor] = field(default_factory=dict)  # workspaces of caches that several layers read
    # retention, state space:
    chunks: Optional[torch.Tensor] = None  # [4, m]: pieces of at most 64 tokens of portions of several tokens: first row, tokens (0 = unused), first position, sequence slot
    n_chunks: int = 0  # at most that many of them are in use
    first_chunk: Optional[torch.Tensor] = None  # [n]: a portion's first piece

    @property
    def rows(self) -> int:
        return self.tokens.numel()


def head_pads(dim: int, vdim: int, dtype: torch.dtype) -> Tuple[int, int]:
    """Elements a cache row takes for keys / values of these sizes."""
    return dim, vdim


def cache_pads(m: Any, dtype: torch.dtype, block_size: int = 16) -> Tuple[int, ...]:
    """Elements per token and head of each of a branch's paged arrays (none: the branch has a state instead)."""
    return (m.kv_rank + m.rot_dim,) if isinstance(m, LatentSpec) else head_pads(m.dim, m.vdim, dtype) if isinstance(m, AttentionSpec) else ()


Join = Optional[Tuple[Optional[torch.Tensor], torch.Tensor]]  # what the stream takes between two layers: rows (or none) and a vector


def embed_stream(table: torch.Tensor, tokens: torch.Tensor, feed: torch.Tensor, prev_ids: torch.Tensor, ld: int, scale: float = 1.0, positions: Optional[torch.Tensor] = None,
                 keep: bool = False) -> Tuple[torch.Tensor, torch.Tensor, Optional[torch.Tensor]]:
    """(stream, the first product's input, a copy of the stream if ``keep``): embedding rows times ``scale``, with ``positions`` plus
    sin / cos of position * 10000^(-2i / width) in columns 2i / 2i + 1."""
    from .torch_ops import embed_tokens

    width = table.shape[1]
    x = embed_tokens(table, tokens, feed, prev_ids).float() * scale
    if positions is not None:
        i = torch.arange(width, dtype=torch.float64, device=x.device)
        ang = positions.double()[:, None] * 10000.0 ** (-2.0 * torch.div(i, 2, rounding_mode="floor") / width)
        x = x + torch.where(i % 2 == 0, ang.sin(), ang.cos()).float()
    x = F.pad(x, (0, ld - width))
    return x, x.to(table.dtype), x.clone() if keep else None


def _unit(v: torch.Tensor, eps: float) -> torch.Tensor:
    return v / torch.sqrt(v.pow(2).mean(-1, keepdim=True) + eps)


def _gain(g: torch.Tensor, width: int) -> torch.Tensor:
    """A norm's gains: one for all columns, or one per column (padded)."""
    return g if g.numel() == 1 else g[:width]


def stream_norm(x: torch.Tensor, join: Join, g: Optional[torch.Tensor], eps: float, width: int, dtype: torch.dtype) -> torch.Tensor:
    """The stream takes ``join``, in place; returns the next product's input: g * unit(x), or without ``g`` the stream itself."""
    if join is not None:
        x += join[1] if join[0] is None else join[0] + join[1]
    if g is None:
        return x.to(dtype)
    return F.pad(_gain(g, width) * _unit(x[:, :width], eps), (0, x.shape[1] - width)).to(dtype)


def gated_residual(x: torch.Tensor, y: torch.Tensor, bias: Optional[torch.Tensor], gate: Optional[torch.Tensor], gate_bias: Optional[torch.Tensor], g: torch.Tensor, mult: float, eps: float,
                   width: int, dtype: torch.dtype, next_g: Optional[torch.Tensor] = None, join: Join = None) -> torch.Tensor:
    """x += mult * g * unit((y + bias) * sigmoid(gate + gate_bias)) over the first ``width`` columns, in place (no gate: factor 1), then
    :func:`stream_norm` with ``join`` and ``next_g``.  Gains: one number or one per column."""
    r = y[:, :width].float()
    if bias is not None:
        r = r + bias[:width]
    if gate is not None:
        r = r * torch.sigmoid(gate[:, :width].float() + gate_bias[:width])
    x[:, :width] += mult * _gain(g, width) * _unit(r, eps)
    return stream_norm(x, join, next_g, eps, width, dtype)


def parallel_residual(x: torch.Tensor, y: Optional[torch.Tensor], bias: Optional[torch.Tensor], y2: Optional[torch.Tensor], g: torch.Tensor, g2: Optional[torch.Tensor], eps: float, width: int,
                      dtype: torch.dtype) -> Tuple[torch.Tensor, Optional[torch.Tensor]]:
    """x += y + bias + y2 (whichever are given), in place; returns g * unit(x) and g2 * unit(x) (no ``g2``: None), the next products' inputs."""
    for r in (y, bias, y2):
        if r is not None:
            x[:, :width] += r[..., :width].float()
    return stream_norm(x, None, g, eps, width, dtype), None if g2 is None else stream_norm(x, None, g2, eps, width, dtype)


def all_streams(n: int, device: Any) -> torch.Tensor:
    """Weights that read the sum of all streams."""
    return torch.ones(n, device=device)


def split_streams(e: torch.Tensor, n: int, read: torch.Tensor, g: torch.Tensor, eps: float, width: int, dtype: torch.dtype) -> Tuple[torch.Tensor, torch.Tensor]:
    """(streams [T, n, ld], all equal to the rows ``e``; the first sublayer's input)."""
    x = e[:, None].repeat(1, n, 1)
    return x, _read_streams(x, read, g, eps, width, dtype)


def _read_streams(x: torch.Tensor, read: torch.Tensor, g: torch.Tensor, eps: float, width: int, dtype: torch.dtype) -> torch.Tensor:
    return stream_norm((x * read[:, None]).sum(1), None, g, eps, width, dtype)


def hyper_residual(x: torch.Tensor, y: torch.Tensor, h: HyperWeights, read: torch.Tensor, g: torch.Tensor, eps: float, width: int, dtype: torch.dtype) -> torch.Tensor:
    """Every stream becomes sum_s mix[s, t] x_s + out[t] y, in place; returns g * unit(sum_t read[t] x_t), the next product's input."""
    x.copy_(torch.einsum("st,bsc->btc", h.mix, x) + h.out[:, None] * y[:, None].float())
    return _read_streams(x, read, g, eps, width, dtype)


def softcap(logits: torch.Tensor, cap: float) -> None:
    """cap * tanh(logits / cap), in place."""
    logits.copy_(cap * torch.tanh(logits.float() / cap))


def _rotate_neighbours(x: torch.Tensor, cos: torch.Tensor, sin: torch.Tensor) -> torch.Tensor:
    u, v = x[..., 0::2], x[..., 1::2]
    return torch.stack((u * cos - v * sin, v * cos + u * sin), -1).flatten(-2)


def _rotate(x: torch.Tensor, cos: torch.Tensor, sin: torch.Tensor, dims: int) -> torch.Tensor:
    if dims == 0:
        return x
    u, v = x[..., : dims // 2], x[..., dims // 2 : dims]
    c, s = cos[:, None, :], sin[:, None, :]
    return torch.cat((u * c - v * s, v * c + u * s, x[..., dims:]), -1)


def attention(m: AttentionSpec, w: AttentionWeights, scale: float, eps: float, proj: torch.Tensor, mix: torch.Tensor, cache: Tuple[torch.Tensor, torch.Tensor], rot: Tuple[torch.Tensor, torch.Tensor],
              st: Step) -> None:
    """Writes the step's keys and values into the paged cache and ``scale`` times the gated head outputs into ``mix``."""
    t = st.rows
    kc, vc = cache
    bs = kc.shape[2]
    nq, nk = m.heads * m.dim, m.kv_heads * m.dim
    q = proj[:, w.q_off : w.q_off + nq].float() + w.bias[:nq]
    k = proj[:, w.k_off : w.k_off + nk].float() + w.bias[nq : nq + nk]
    v = proj[:, w.v_off : w.v_off + m.kv_heads * m.vdim].float() + w.bias[nq + nk :]
    q, k, v = q.view(t, m.heads, m.dim), k.view(t, m.kv_heads, m.dim), v.view(t, m.kv_heads, m.vdim)
    pos = st.positions.long()
    cos, sin = (None, None) if m.rot_dims == 0 else (rot[0][pos], rot[1][pos])
    q = _rotate(q / torch.sqrt(q.pow(2).mean(-1, keepdim=True) + eps) * w.q_norm, cos, sin, m.rot_dims)
    k = _rotate(k / torch.sqrt(k.pow(2).mean(-1, keepdim=True) + eps) * w.k_norm, cos, sin, m.rot_dims)
    rows = (st.slots >= 0).nonzero().view(-1)
    slot = st.slots[rows].long()
    kc[slot // bs, :, slot % bs] = k[rows].to(kc.dtype)
    vc[slot // bs, :, slot % bs] = v[rows].to(vc.dtype)
    q = q.to(proj.dtype).float()
    rep = m.heads // m.kv_heads
    gates = torch.sigmoid(proj[:, w.g_off : w.g_off + m.gates].float()).view(t, m.heads, -1) if m.gates else torch.ones(t, 1, 1)
    for i in rows.tolist():
        p = int(pos[i])
        first = p - p % m.chunk if m.chunk else max(0, p - m.window + 1) if m.window else 0
        keys = torch.cat((torch.arange(min(m.keep, first)), torch.arange(first, p + 1)))
        blk = st.block_tables[int(st.tok_seq[i])].long()[keys // bs]
        ks = kc[blk, :, keys % bs].float()  # [keys, kv heads, dim]
        vs = vc[blk, :, keys % bs].float()
        s = torch.einsum("grd,kgd->grk", q[i].view(m.kv_heads, rep, m.dim), ks) * m.scale
        if w.rel is not None:
            s = s + w.rel[:, (p - keys).clamp(max=w.rel.shape[1] - 1)].view(s.shape)
        if w.sink is not None:  # (a key of its own, whose value is nothing)
            s = torch.cat((s, w.sink.view(m.kv_heads, rep, 1)), -1)
        o = torch.einsum("grk,kgd->grd", torch.softmax(s, -1)[..., : len(keys)], vs).reshape(m.heads, m.vdim)
        mix[i, w.o_off : w.o_off + m.heads * m.vdim] = (o * gates[i] * scale).reshape(-1).to(mix.dtype)


def latent_attention(m: LatentSpec, w: LatentWeights, scale: float, eps: float, proj: torch.Tensor, mix: torch.Tensor, cache: torch.Tensor, st: Step,
                     rot: Optional[Tuple[torch.Tensor, torch.Tensor]] = None) -> None:
    """Writes the step's latents (with their rotated key parts, unless the cache is another layer's) into the paged cache and ``scale``
    times the gated head outputs into ``mix``.  Scores and sums are taken in the latent space: q . (W_uk c) = (W_uk^T q) . c, and W_uv
    goes onto the weighted sum of the latents."""
    t, bs, rank = st.rows, cache.shape[2], m.kv_rank
    rows = (st.slots >= 0).nonzero().view(-1)
    cos, sin = (None, None) if rot is None else (rot[0][st.positions.long()], rot[1][st.positions.long()])
    if m.kv_from < 0:
        c = _unit(proj[:, w.c_off : w.c_off + rank].float(), eps) * w.c_norm[:rank]
        if m.rot_dim:
            c = torch.cat((c, _rotate_neighbours(proj[:, w.kr_off : w.kr_off + m.rot_dim].float(), cos, sin)), -1)
        slot = st.slots[rows].long()
        cache[slot // bs, 0, slot % bs] = c[rows].to(cache.dtype)
    q = proj[:, w.q_off : w.q_off + m.heads * w.dkp].float().view(t, m.heads, w.dkp)
    q = torch.einsum("thd,hrd->thr", q, w.absorb.float())
    if m.rot_dim:
        qr = proj[:, w.r_off : w.r_off + m.heads * m.rot_dim].float().view(t, m.heads, m.rot_dim)
        q = torch.cat((q, _rotate_neighbours(qr, cos[:, None], sin[:, None])), -1)
    gates = torch.sigmoid(proj[:, w.g_off : w.g_off + m.gates].float()).view(t, m.heads, -1)
    for i in rows.tolist():
        p = int(st.positions[i])
        keys = torch.arange(max(0, p - m.window + 1) if m.window else 0, p + 1)
        cs = cache[st.block_tables[int(st.tok_seq[i])].long()[keys // bs], 0, keys % bs].float()
        o = torch.softmax(q[i] @ cs.T * m.scale, -1) @ cs[:, :rank]
        o = torch.einsum("hvr,hr->hv", w.up.float(), o)
        mix[i, w.o_off : w.o_off + m.heads * m.vdim] = (o * gates[i] * scale).reshape(-1).to(mix.dtype)


def choose_experts(m: MoeSpec, w: MoeWeights, h: torch.Tensor) -> Tuple[torch.Tensor, torch.Tensor]:
    """([T, top] experts, their weights)."""
    z = h.float() @ w.router[: m.experts].float().T
    if w.bias is not None:
        z = z + w.bias
    if m.scores == "chosen":
        idx = torch.topk(z + w.correction, m.top, dim=-1).indices
        return idx, torch.softmax(z.gather(-1, idx), -1) * m.scale
    s = torch.softmax(z, -1) if m.scores == "softmax" else torch.sigmoid(z)
    idx = torch.topk(s + w.correction, m.top, dim=-1).indices
    return idx, s.gather(-1, idx) * m.scale


def experts(m: MoeSpec, w: MoeWeights, h: torch.Tensor, st: Step) -> torch.Tensor:
    """Weighted sum of the chosen experts' outputs, and the shared expert's, fp32 [T, ld]."""
    from kvmini.models.llama import GU_GROUP

    idx, wt = choose_experts(m, w, h)
    idx = torch.where(st.slots[:, None] >= 0, idx, torch.full_like(idx, -1))  # (padding rows choose nobody)
    out = torch.zeros((h.shape[0], h.shape[1]), dtype=torch.float32, device=h.device)
    for e in idx.unique().tolist():
        if e < 0:
            continue
        t, k = (idx == e).nonzero(as_tuple=True)
        if not m.gated:
            out[t] += F.linear(F.relu(F.linear(h[t], w.gate_up[e]).float()).square().to(h.dtype), w.down[e]).float() * wt[t, k][:, None]
            continue
        gu = F.linear(h[t], w.gate_up[e]).view(len(t), w.ffp // GU_GROUP, 2, GU_GROUP).float()
        limit, a, b = m.glu
        g, u = gu[:, :, 0].clamp(max=limit), gu[:, :, 1].clamp(-limit, limit)
        act = (g * torch.sigmoid(a * g) * (u + b)).reshape(len(t), w.ffp).to(h.dtype)
        out[t] += F.linear(act, w.down[e]).float() * wt[t, k][:, None]
    if m.shared_ff:
        from .torch_ops import linear_relu2, linear_swiglu

        y = F.linear((linear_swiglu if m.gated else linear_relu2)(h, w.shared_gate_up), w.shared_down).float()
        if not m.shared_gate:
            return out + y
        out += torch.sigmoid(h.float() @ w.router[m.experts].float())[:, None] * y
    return out


class Retention:
    """A retention branch with its per-sequence state (fp32 [slots, heads, dim, vdim], padded to whole tiles with zeros)."""

    def __init__(self, m: RetentionSpec, w: RetentionWeights, scale: float, eps: float, state: torch.Tensor, rot: Tuple[torch.Tensor, torch.Tensor]):
        self.m, self.w, self.scale, self.eps, self.state, self.rot = m, w, scale, eps, state, rot

    def run(self, proj: torch.Tensor, mix: torch.Tensor, st: Step) -> None:
        m, w = self.m, self.w
        qk, nv = m.heads * m.dim, m.heads * m.vdim
        decay = torch.exp2(w.log2_decay)[:, None, None]
        for row, n, p0, slot, _tile in st.portions.t().tolist():
            if n == 0:
                continue
            r = slice(row, row + n)
            pos = st.positions[r].long()
            q, k = (_rotate(proj[r, o : o + qk].float().view(n, m.heads, m.dim), self.rot[0][pos], self.rot[1][pos], m.rot_dims) for o in (w.q_off, w.k_off))
            k, v = k * m.dim ** -0.5, proj[r, w.v_off : w.v_off + nv].float().view(n, m.heads, m.vdim)
            s = self.state[slot, :, : m.dim, : m.vdim] if p0 > 0 else torch.zeros(m.heads, m.dim, m.vdim, device=proj.device)
            os = []
            for i in range(n):
                s = decay * s + k[i][:, :, None] * v[i][:, None, :]
                os.append(torch.einsum("hdv,hd->hv", s, q[i]))
            self.state[slot, :, : m.dim, : m.vdim] = s
            o = self.scale * _unit(torch.stack(os), self.eps) * F.silu(proj[r, w.g_off : w.g_off + nv].float()).view(n, m.heads, m.vdim)
            mix[r, w.o_off : w.o_off + nv] = o.reshape(n, nv).to(mix.dtype)


class DeltaState:
    """A delta-rule branch with its per-sequence state (``state`` fp32 [slots, heads, dim, vdim]; ``ring`` [slots, taps, channels]:
    convolution inputs, position p at p % taps)."""

    def __init__(self, m: DeltaSpec, w: DeltaWeights, scale: float, eps: float, state: torch.Tensor, ring: torch.Tensor):
        self.m, self.w, self.scale, self.eps, self.state, self.ring = m, w, scale, eps, state, ring

    def run(self, proj: torch.Tensor, low: torch.Tensor, mix: torch.Tensor, st: Step) -> None:
        m, w = self.m, self.w
        kv, d, dv = m.kv_heads, m.dim, m.vdim
        nq, nv, rep = kv * d, m.heads * dv, m.heads // kv
        portions: List[Any] = [(r, n, p, s) for r, n, p, s, _tile in st.portions.t().tolist() if n > 0]
        for row, n, p0, slot in portions:
            r = slice(row, row + n)
            xin = torch.cat((proj[r, w.q_off : w.q_off + nq], proj[r, w.k_off : w.k_off + nq], proj[r, w.v_off : w.v_off + nv]), -1)
            past = [self.ring[slot, p % m.taps] if p >= 0 else torch.zeros_like(self.ring[slot, 0]) for p in range(p0 - m.taps + 1, p0)]
            ext = torch.cat((torch.stack(past), xin)).float() if past else xin.float()
            y = F.silu(sum(w.conv[j] * ext[j : j + n] for j in range(m.taps)))
            q, k, v = y[:, :nq].view(n, kv, d), y[:, nq : 2 * nq].view(n, kv, d), y[:, 2 * nq :].view(n, m.heads, dv)
            q = q / torch.sqrt(q.pow(2).sum(-1, keepdim=True) + 1e-6) * d ** -0.5
            k = k / torch.sqrt(k.pow(2).sum(-1, keepdim=True) + 1e-6)
            q, k = q.repeat_interleave(rep, 1), k.repeat_interleave(rep, 1)
            beta = torch.sigmoid(proj[r, w.b_off : w.b_off + m.heads].float())
            z = low[r, w.z_off : w.z_off + m.heads * d].float() + w.dt_bias
            decay = torch.exp(-torch.exp(w.a_log)[:, None] * F.softplus(z, threshold=50.0).view(n, m.heads, d))
            s = self.state[slot] if p0 > 0 else torch.zeros_like(self.state[slot])
            os = []
            for i in range(n):
                s = decay[i][:, :, None] * s
                u = beta[i][:, None] * (v[i] - torch.einsum("hdv,hd->hv", s, k[i]))
                s = s + k[i][:, :, None] * u[:, None, :]
                os.append(torch.einsum("hdv,hd->hv", s, q[i]))
            self.state[slot] = s
            for i in range(max(0, n - m.taps), n):
                self.ring[slot, (p0 + i) % m.taps] = xin[i]
            o = torch.stack(os)
            gate = torch.sigmoid(low[r, w.gate_off : w.gate_off + nv].float()).view(n, m.heads, dv)
            o = self.scale * o / torch.sqrt(o.pow(2).mean(-1, keepdim=True) + self.eps) * w.norm * gate
            mix[r, w.o_off : w.o_off + nv] = o.reshape(n, nv).to(mix.dtype)


class StateSpace:
    """A state-space branch with its per-sequence memory (``state`` fp32 [slots, heads, dim, vdim], padded to whole tiles with zeros; ``ring``
    [slots, taps, channels]: convolution inputs, position p at p % taps)."""

    def __init__(self, m: StateSpaceSpec, w: StateSpaceWeights, scale: float, eps: float, state: torch.Tensor, ring: torch.Tensor):
        self.m, self.w, self.scale, self.eps, self.state, self.ring = m, w, scale, eps, state, ring

    def run(self, proj: torch.Tensor, mix: torch.Tensor, st: Step) -> None:
        m, w = self.m, self.w
        gn, rep = m.groups * m.dim, m.heads // m.groups
        for row, n, p0, slot, _tile in st.portions.t().tolist():
            if n == 0:
                continue
            r = slice(row, row + n)
            xin = proj[r, w.x_off : w.x_off + m.channels]
            past = [self.ring[slot, p % m.taps] if p >= 0 else torch.zeros_like(self.ring[slot, 0]) for p in range(p0 - m.taps + 1, p0)]
            ext = torch.cat((torch.stack(past), xin)).float() if past else xin.float()
            for i in range(max(0, n - m.taps), n):
                self.ring[slot, (p0 + i) % m.taps] = xin[i]
            y = F.silu(sum(w.conv[j] * ext[j : j + n] for j in range(m.taps)) + w.conv_bias).to(proj.dtype).float()
            x, b, c = y[:, : m.inner].view(n, m.heads, m.vdim), *(y[:, o : o + gn].view(n, m.groups, m.dim).repeat_interleave(rep, 1) for o in (m.inner, m.inner + gn))
            dt = F.softplus(proj[r, w.dt_off : w.dt_off + m.heads].float() + w.dt_bias, threshold=50.0)
            decay = torch.exp(-torch.exp(w.a_log) * dt)
            s = self.state[slot, :, : m.dim, : m.vdim] if p0 > 0 else torch.zeros(m.heads, m.dim, m.vdim, device=proj.device)
            os = []
            for i in range(n):
                s = decay[i][:, None, None] * s + (dt[i][:, None] * b[i])[:, :, None] * x[i][:, None, :]
                os.append(torch.einsum("hdv,hd->hv", s, c[i]) + w.skip[:, None] * x[i])
            self.state[slot, :, : m.dim, : m.vdim] = s
            o = torch.stack(os).view(n, m.inner) * F.silu(proj[r, w.z_off : w.z_off + m.inner].float())
            o = _unit(o.view(n, m.norm_groups, -1), self.eps).view(n, m.inner) * w.norm * self.scale
            mix[r, w.o_off : w.o_off + m.inner] = o.to(mix.dtype)
