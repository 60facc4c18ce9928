"""Sequence mixers and experts on the hand-written gfx950 kernels (``csrc/mixer_kernels.hip``, ``chunk_attention.hip``,
``delta_rule.hip``, ``latent_attention.hip``, ``retention.hip``, ``state_space.hip``, ``experts.hip``, the grouped form of ``wide_gemm.hip``); call surface of :mod:`kvmini.ops.torch_mixers`."""

from __future__ import annotations

import functools
import math
from typing import Any, Optional, Tuple

import torch

from kvmini.models.hybrid import (AttentionSpec, AttentionWeights, DeltaSpec, DeltaWeights, HyperWeights, LatentSpec, LatentWeights, Layout, MoeSpec, MoeWeights, RetentionSpec,
                                  RetentionWeights, StateSpaceSpec, StateSpaceWeights, round_up)

from . import native
from .hip_ops import PackedLinear, Partial, _num_cus
from .torch_mixers import Join, Step

__all__ = ["Step", "head_pads", "cache_pads", "layout", "embed_stream", "stream_norm", "gated_residual", "all_streams", "split_streams", "hyper_residual", "parallel_residual", "softcap", "attention", "latent_attention", "experts", "shared_expert", "with_shared", "decode_plan", "DeltaState", "Retention", "StateSpace"]


def head_pads(dim: int, vdim: int, dtype: torch.dtype) -> Tuple[int, int]:
    """bf16: the next sizes the matrix-core kernels are built for; sizes beyond them and fp32 go through the row kernel
    (multiples of four)."""
    if dtype == torch.bfloat16:
        if max(dim, vdim) <= 128:
            return (64 if dim <= 64 else 128), (64 if vdim <= 64 else 128)
        if max(dim, vdim) <= 256:
            return 256, 256
    return -(-dim // 4) * 4, -(-vdim // 4) * 4


def key_value_pads(m: AttentionSpec, dtype: torch.dtype, block_size: int = 16) -> Optional[Tuple[int, int]]:
    """(value, rotated part) of a cache row that is key and value at once, where the kernels have that form and it saves memory: bf16, values
    that are the keys as projected."""
    if block_size < 16 or block_size & (block_size - 1) or not m.key_values or dtype != torch.bfloat16 or m.dim > 256 or (m.rel and m.rot_dims):
        return None
    dim, rot = (64 if m.dim <= 64 else 128 if m.dim <= 128 else 256), 0 if m.rot_dims == 0 else 32 if m.rot_dims <= 32 else 64
    return (dim, rot) if m.rot_dims <= rot < dim else None


class RowLayout(Layout):
    """fp32, and sizes beyond the matrix-core kernels: row-major, head sizes in fours."""

    def latent_pads(self, m: LatentSpec) -> Tuple[int, int, int]:
        return round_up(m.dim, 4), round_up(m.vdim, 4), round_up(m.kv_rank, 4)

    def rot_pad(self, m: LatentSpec) -> int:
        return round_up(m.rot_dim, 4)


class FragmentLayout(RowLayout):
    """bf16: fragment order of the matrix instructions, latent attention padded to the sizes its kernels are built for."""

    def __call__(self, w: torch.Tensor) -> Any:
        return PackedLinear(w)

    def out_rows(self, n: int) -> int:
        """Widths the tiled GEMM has its large tiles for, where that costs few rows."""
        return next((p for p in (round_up(n, 256), round_up(n, 128)) if p - n <= n // 20), round_up(n, 64))

    def expands(self, m: LatentSpec) -> bool:
        return max(m.dim, m.vdim) <= 256 and m.kv_rank <= 512 and m.rot_dim <= 64

    def latent_pads(self, m: LatentSpec) -> Tuple[int, int, int]:
        """(The latent's size depends on nothing but its own: layers of different heads may share a cache.)"""
        size = lambda n: 64 if n <= 64 else 128 if n <= 128 else 256  # noqa: E731
        dim, vdim, rank = super().latent_pads(m)
        if m.kv_rank <= 512:
            rank = 128 if m.kv_rank <= 128 else 256 if m.kv_rank <= 256 else 512
        return (size(m.dim), size(m.vdim), rank) if self.expands(m) else (dim, vdim, rank)

    def rot_pad(self, m: LatentSpec) -> int:
        return 64 if 0 < m.rot_dim <= 64 else super().rot_pad(m)

    @staticmethod
    def _pack(w: torch.Tensor) -> torch.Tensor:
        return native().pack_weight(w.reshape(-1, w.shape[-1]).contiguous()).view(w.shape)

    def heads(self, w: torch.Tensor, m: LatentSpec) -> torch.Tensor:
        return self._pack(w) if self.expands(m) else w

    def experts(self, w: torch.Tensor) -> torch.Tensor:
        return self._pack(w)

    def expert_width(self, ff: int, gated: bool = True) -> int:
        return round_up(ff, 64 if gated else 128)

    def router(self, w: torch.Tensor) -> torch.Tensor:
        return self._pack(torch.nn.functional.pad(w, (0, 0, 0, -w.shape[0] % 16)))


def layout(dtype: torch.dtype) -> Layout:
    return FragmentLayout() if dtype == torch.bfloat16 else RowLayout()


def cache_pads(m: Any, dtype: torch.dtype, block_size: int = 16) -> Tuple[int, ...]:
    if isinstance(m, LatentSpec):
        lay = layout(dtype)
        return (lay.latent_pads(m)[2] + lay.rot_pad(m),)
    if isinstance(m, AttentionSpec):
        one = key_value_pads(m, dtype, block_size)
        return head_pads(m.dim, m.vdim, dtype) if one is None else (sum(one), 2)  # (behind the rows: the fp32 factors that norm the keys)
    return ()


@functools.lru_cache(maxsize=None)
def _sine_turns(width: int, device: torch.device) -> torch.Tensor:
    """10000^(-2i / width) / 2 pi, the sines' frequencies in turns per position, as sums of two floats, [(width + 1) / 2, 2]."""
    f = 10000.0 ** (-2.0 * torch.arange((width + 1) // 2, dtype=torch.float64) / width) / (2 * math.pi)
    hi = f.float()
    return torch.stack((hi, (f - hi.double()).float()), 1).contiguous().to(device)


def embed_stream(table: torch.Tensor, tokens: torch.Tensor, feed: torch.Tensor, prev_ids: torch.Tensor, ld: int, scale: float = 1.0, positions: Optional[torch.Tensor] = None,
                 keep: bool = False) -> Tuple[torch.Tensor, torch.Tensor, Optional[torch.Tensor]]:
    t = tokens.numel()
    x = torch.empty((t, ld), dtype=torch.float32, device=table.device)
    copy = torch.empty_like(x) if keep else None
    xb = torch.empty((t, ld), dtype=table.dtype, device=table.device)
    native().embed_stream(table, tokens, feed, prev_ids, x, xb, copy, scale, positions, None if positions is None else _sine_turns(table.shape[1], table.device))
    return x, xb, copy


class ExpertRows:
    """A mixture's result before the weighted sum: rows ``[T * top, ld]`` and weights ``[T, top]`` (0: the row was never written); a
    shared expert's rows (or split-K partial sums) and their factors ``[T]``."""

    __slots__ = ("rows", "weights", "shared", "shared_gate")

    def __init__(self, rows: torch.Tensor, weights: torch.Tensor, shared: Any = None, shared_gate: Optional[torch.Tensor] = None):
        self.rows, self.weights, self.shared, self.shared_gate = rows, weights, shared, shared_gate


def _slabs(y: Any) -> Any:
    return y.slabs if isinstance(y, Partial) else y


@functools.lru_cache(maxsize=None)
def all_streams(n: int, device: torch.device) -> torch.Tensor:
    return torch.ones(n, dtype=torch.float32, device=device)


def split_streams(e: torch.Tensor, n: int, read: torch.Tensor, g: torch.Tensor, eps: float, width: int, dtype: torch.dtype) -> Tuple[torch.Tensor, torch.Tensor]:
    x = torch.empty((e.shape[0], n, e.shape[1]), dtype=torch.float32, device=e.device)
    xb = torch.empty(e.shape, dtype=dtype, device=e.device)
    native().hyper_residual(x, xb, None, None, None, None, None, None, read, g, e, eps, width)
    return x, xb


def hyper_residual(x: torch.Tensor, y: Any, h: HyperWeights, read: torch.Tensor, g: torch.Tensor, eps: float, width: int, dtype: torch.dtype) -> torch.Tensor:
    """``y`` may be split-K partial sums or experts' rows: they are summed on the way in."""
    xb = torch.empty((x.shape[0], x.shape[2]), dtype=dtype, device=x.device)
    weights = shared = gate = None
    if isinstance(y, ExpertRows):
        y, weights, shared, gate = y.rows, y.weights, y.shared, y.shared_gate
    native().hyper_residual(x, xb, _slabs(y), weights, _slabs(shared), gate, h.mix, h.out, read, g, None, eps, width)
    return xb


def parallel_residual(x: torch.Tensor, y: Any, bias: Optional[torch.Tensor], y2: Optional[ExpertRows], g: torch.Tensor, g2: Optional[torch.Tensor], eps: float, width: int,
                      dtype: torch.dtype) -> Tuple[torch.Tensor, Optional[torch.Tensor]]:
    """``y`` may be split-K partial sums: they and experts' rows are summed on the way in."""
    xb = torch.empty(x.shape, dtype=dtype, device=x.device)
    xb2 = None if g2 is None else torch.empty_like(xb)
    rows, weights, shared = (None, None, None) if y2 is None else (y2.rows, y2.weights, y2.shared)
    native().parallel_residual(x, xb, xb2, _slabs(y), rows, weights, _slabs(shared), bias, g, g2, eps, width)
    return xb, xb2


def softcap(logits: torch.Tensor, cap: float) -> None:
    native().softcap(logits, cap)


def gated_residual(x: torch.Tensor, y: Any, bias: Optional[torch.Tensor], gate: Any, gate_bias: Optional[torch.Tensor], g: Optional[torch.Tensor], mult: float, eps: float, width: int,
                   dtype: torch.dtype, next_g: Optional[torch.Tensor] = None, join: Join = None) -> torch.Tensor:
    """``y`` and ``gate`` may be split-K partial sums, ``y`` experts' rows: they are summed on the way in."""
    xb = torch.empty(x.shape, dtype=dtype, device=x.device)
    weights = None
    if isinstance(y, ExpertRows):
        y, weights = y.rows, y.weights
    native().gated_residual(x, xb, _slabs(y), weights, bias, _slabs(gate), gate_bias, g, next_g,
                            None if join is None else join[0], None if join is None else join[1], mult, eps, width)
    return xb


def stream_norm(x: torch.Tensor, join: Join, g: Optional[torch.Tensor], eps: float, width: int, dtype: torch.dtype) -> torch.Tensor:
    return gated_residual(x, None, None, None, None, None, 1.0, eps, width, dtype, g, join)


def attention(m: AttentionSpec, w: AttentionWeights, scale: float, eps: float, proj: torch.Tensor, mix: torch.Tensor, cache: Tuple[torch.Tensor, torch.Tensor], rot: Tuple[torch.Tensor, torch.Tensor],
              st: Step) -> None:
    C = native()
    kc, vc = cache
    one = vc.shape[3] == 2  # (one row is key and value: the second array holds the keys' factors)
    if one:
        vc = vc.view(torch.float32)
    tiled = one or proj.dtype == torch.bfloat16 and C.chunk_prefill_supported(kc.shape[3], vc.shape[3]) and kc.shape[2] >= 16 and kc.shape[2] & (kc.shape[2] - 1) == 0
    q, see = None, (m.chunk, m.window, m.keep, w.sink, w.rel)
    gates = ("none", "head", "element").index(m.gate)
    if not (tiled and st.decode_only):
        q = torch.empty((st.rows, m.heads, kc.shape[3]), dtype=proj.dtype, device=proj.device)
        write = (proj, w.q_off, w.k_off), (w.bias, w.q_norm, w.k_norm, st.positions, st.slots, rot[0], rot[1], m.rot_dims, q, kc, vc, m.dim)
        if one:
            C.key_value_write(*write[0], *write[1], eps)
        else:
            C.norm_rope_write(*write[0], w.v_off, *write[1], m.vdim, eps)
    if not tiled:
        C.row_attention(q, kc, vc, st.block_tables, st.tok_seq, st.positions, st.slots, proj, w.g_off, gates, mix, w.o_off, m.vdim, *see, m.scale, scale, None, -1)
        return
    if not st.decode_only:
        C.chunk_prefill(q, kc, vc, st.block_tables, st.blocks, st.n_blocks, proj, w.g_off, gates, mix, w.o_off, m.vdim, *see, m.scale, scale)
    waves, shares = decode_plan(st.singles.numel(), m.kv_heads * -(-(m.heads // m.kv_heads) // 16), st.long)
    C.chunk_decode(q, proj, w.q_off, w.k_off, w.v_off, w.bias, w.q_norm, w.k_norm, rot[0], rot[1], m.rot_dims, eps, kc, vc, st.block_tables, st.singles, st.tok_seq, st.positions, st.slots,
                   w.g_off, gates, mix, w.o_off, m.heads, m.dim, m.vdim, *see, m.scale, scale, waves, shares)


def decode_plan(rows: int, groups: int, long: bool) -> Tuple[int, int]:
    """(waves per workgroup, workgroups per row and key head) of the decode attention kernel: eight waves while the grid does not
    fill the CUs, and for long contexts several workgroups per row (their partial results cost a second launch)."""
    cus = _num_cus()
    waves = 8 if rows * groups <= cus else 4
    return waves, max(1, min(16, 2 * cus // (rows * groups))) if long else 1


def latent_attention(m: LatentSpec, w: LatentWeights, scale: float, eps: float, proj: torch.Tensor, mix: torch.Tensor, cache: torch.Tensor, st: Step,
                     rot: Optional[Tuple[torch.Tensor, torch.Tensor]] = None) -> None:
    C = native()
    cos, sin = rot or (None, None)
    each, own = m.gate == "element", m.kv_from < 0
    norm = w.c_norm if own else None
    turns = (w.kr_off, cos, sin, m.heads, w.r_off)
    if w.expand is None:  # every row in the latent space, one by one
        row = w.rkp + w.rtp
        q = torch.empty((st.rows, m.heads, row), dtype=proj.dtype, device=proj.device)
        o = torch.empty((st.rows, m.heads * w.rkp), dtype=proj.dtype, device=proj.device)
        if own or m.rot_dim:
            C.latent_write(proj, w.c_off, norm, st.slots, st.positions, cache, m.kv_rank, w.rkp, eps, *turns, q.view(st.rows, -1), w.rkp, row)
        C.head_rows(proj, w.q_off, w.dkp, w.absorb, w.rkp, None, 0, False, q.view(st.rows, -1), 0, row, 1.0, st.slots)
        C.row_attention(q, cache, cache, st.block_tables, st.tok_seq, st.positions, st.slots, None, 0, 0, o, 0, w.rkp, 0, m.window, 0, None, None, m.scale, 1.0, None, -1)
        C.head_rows(o, 0, w.rkp, w.up, m.vdim, proj, w.g_off, each, mix, w.o_off, m.vdim, scale, st.slots)
        return
    if not st.decode_only:
        from .hip_ops import linear

        if own or m.rot_dim:  # (the queries' rotated parts turn where they are)
            C.latent_write(proj, w.c_off, norm, st.slots, st.positions, cache, m.kv_rank, w.rkp, eps, *turns, proj if m.rot_dim else None, w.r_off, w.rtp)
        ws = st.gathered.get(cache.data_ptr())
        if ws is None:  # (layers that share a cache share what was gathered from it)
            ws = st.gathered[cache.data_ptr()] = torch.empty((st.span_rows, w.rkp + w.rtp), dtype=proj.dtype, device=proj.device)
            C.latent_gather(cache, st.spans, st.block_tables, ws)
        C.latent_prefill(proj, w.q_off, w.r_off, w.g_off, each, linear(ws[:, : w.rkp], w.expand), ws[:, w.rkp :] if w.rtp else None, st.latent_blocks, st.n_latent_blocks, mix, w.o_off, m.heads,
                         w.dkp, m.vdim, w.dvp, m.window, m.scale, scale)
    shares, parts = latent_plan(st.singles.numel(), m.heads, w.dvp, m.window, st.long)
    C.latent_rows(proj, w.q_off, w.r_off, w.c_off, w.kr_off, w.g_off, each, w.absorb, w.up, norm, m.kv_rank, eps, cos, sin, cache, own and st.decode_only, st.decode_only, st.block_tables,
                  st.singles, st.tok_seq, st.positions, st.slots, mix, w.o_off, m.vdim, m.window, m.scale, scale, shares, parts)


def latent_plan(rows: int, heads: int, dvp: int, window: int, long: bool) -> Tuple[int, int]:
    """(workgroups per row and group of 16 heads of the latent attention, workgroups per head of the product behind it): what fills
    the CUs, for long contexts; a share should have a block of 16 keys for each of its four waves."""
    cus = _num_cus()
    most = min(16, -(-(window // 16 + 1) // 4)) if window else 16
    shares = max(1, min(most, cus // (rows * -(-heads // 16)))) if long else 1
    return shares, max(1, min(dvp // 64, cus // (heads * -(-rows // 16))))


EXPERT_FEW_ROWS = 128  # up to as many tokens, workgroups look up their experts' rows themselves; beyond, rows are grouped into tiles


def expert_tile(tokens: int, top: int, experts: int) -> int:
    """Rows per tile of the grouped products: what an expert's rows (somewhat more than the mean) fill best.  A tile loads its operands
    once for all its rows, so per row the small ones cost more."""
    mean = tokens * top / experts
    rows = mean + 2.0 * mean ** 0.5
    return min((256, 128, 64), key=lambda t: -(-rows // t) * t * (1.0 + 76.0 / t))


def shared_expert(m: MoeSpec, w: MoeWeights, h: torch.Tensor) -> Any:
    from .hip_ops import linear, linear_relu2, linear_swiglu

    return linear((linear_swiglu if m.gated else linear_relu2)(h, w.shared_gate_up), w.shared_down, allow_slabs=True)


def with_shared(y: ExpertRows, m: MoeSpec, w: MoeWeights, h: torch.Tensor) -> ExpertRows:
    """The chosen experts' rows (of :func:`experts` without the shared one) and the shared expert's, which is computed here."""
    return ExpertRows(y.rows, y.weights, shared_expert(m, w, h), y.shared_gate) if m.shared_ff else y


def experts(m: MoeSpec, w: MoeWeights, h: torch.Tensor, st: Step, shared: bool = True) -> ExpertRows:
    C = native()
    gate_row = m.shared_ff > 0 and m.shared_gate
    idx, wt, gate = C.route(h, w.router, w.correction, st.slots, m.top, ("sigmoid", "softmax", "chosen").index(m.scores), m.scale, gate_row, w.bias)
    t = h.shape[0]
    tile = 0 if h.dtype != torch.bfloat16 or t <= EXPERT_FEW_ROWS else expert_tile(t, m.top, m.experts)
    rows = C.expert_outputs(h, idx, w.gate_up, w.down, m.gated, *m.glu, tile)
    out = ExpertRows(rows, wt, None, gate if gate_row else None)
    return with_shared(out, m, w, h) if shared else out


class DeltaState:
    def __init__(self, m: DeltaSpec, w: DeltaWeights, scale: float, eps: float, state: torch.Tensor, ring: torch.Tensor):
        self.impl = native().DeltaLayer(m.heads, m.kv_heads, m.dim, m.vdim, eps, scale, [w.q_off, w.k_off, w.v_off, w.b_off, w.z_off, w.gate_off, w.o_off], w.conv, w.a_log, w.dt_bias, w.norm, state, ring)
        self.has_step, self.has_tiles = self.impl.has_step(), self.impl.has_tiles()

    def run(self, proj: torch.Tensor, low: torch.Tensor, mix: torch.Tensor, st: Step) -> None:
        per_token = (st.tok_seq, st.positions, st.tok_kind, st.tok_off)
        if self.has_step:  # the rows that are alone
            self.impl.step(proj, low, mix, *per_token, st.singles)
            if st.decode_only:
                return
        # portions: tiles of 16 tokens — or token by token, for key sizes beyond the tile kernels and heads the one-token kernel does not take
        tiles = self.has_step and self.has_tiles
        self.impl.portions(proj, low, mix, *per_token, st.portions, 2 if self.has_step else 1, st.tiles, st.n_tiles if tiles else 0)


class Retention:
    def __init__(self, m: RetentionSpec, w: RetentionWeights, scale: float, eps: float, state: torch.Tensor, rot: Tuple[torch.Tensor, torch.Tensor]):
        self.impl = native().RetentionLayer(m.heads, m.dim, m.vdim, eps, scale, [w.q_off, w.k_off, w.v_off, w.g_off, w.o_off], w.log2_decay, rot[0], rot[1], m.rot_dims, state)
        self.chunked = self.impl.chunked()

    def run(self, proj: torch.Tensor, mix: torch.Tensor, st: Step) -> None:
        per_token = (st.tok_seq, st.positions, st.tok_kind)
        self.impl.step(proj, mix, *per_token, st.singles)  # the rows that are alone
        if not st.decode_only:
            self.impl.portions(proj, mix, *per_token, st.portions, st.chunks, st.n_chunks if self.chunked else 0, st.first_chunk)


class StateSpace:
    def __init__(self, m: StateSpaceSpec, w: StateSpaceWeights, scale: float, eps: float, state: torch.Tensor, ring: torch.Tensor):
        self.impl = native().StateSpaceLayer(m.heads, m.groups, m.dim, m.vdim, m.norm_groups, eps, scale, [w.z_off, w.x_off, w.dt_off, w.o_off], w.conv, w.conv_bias, w.dt_bias, w.a_log, w.skip, w.norm,
                                             state, ring)

    def run(self, proj: torch.Tensor, mix: torch.Tensor, st: Step) -> None:
        self.impl.run(proj, mix, st.tok_seq, st.positions, st.tok_kind, st.tok_off, st.singles, st.portions, st.chunks, 0 if st.decode_only else st.n_chunks, st.first_chunk)
