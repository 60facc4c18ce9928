"""Decoders whose layers mix tokens by attention, by a recurrence, or by several such branches side by side.

A configuration is a list of :class:`LayerSpec`; a layer has one or more *branches* that read the same input
(:class:`AttentionSpec`: softmax attention with its own query / key and value sizes, query / key norm, partial rotation or a
learned distance bias, chunked or windowed visibility, sinks and gates; :class:`LatentSpec`: softmax attention whose keys and values are linear images of one
cached latent vector per token, optionally beside a rotated key part shared by all heads, inside a sliding window or not, with
gates per head or per element, optionally on another layer's latents; :class:`DeltaSpec`: gated delta rule with a decay per key
channel behind short convolutions; :class:`RetentionSpec`: linear attention with a fixed decay per head;
:class:`StateSpaceSpec`: linear attention whose decay and step size per head come from the token) and an optional
feed-forward: a gated MLP or a mixture of experts (:class:`MoeSpec`).  The residual stream is 32-bit.  Four wirings of a
sublayer exist (``HybridConfig.wiring``): ``gated`` — it reads the stream itself, and its result is gated element by element,
normalised with one gain and added; ``sandwich`` — it reads the normalised stream, and its result is normalised and added (gains
per channel on both sides); ``hyper`` — there are several streams, it reads the normalised weighted sum of them, and every
stream becomes a weighted sum of all streams and the result; ``parallel`` — a layer's mixer and feed-forward read the same
stream, each behind a norm of its own, and both results are added to it at once.  A stretch of layers may run several times in a row
(:class:`LoopSpec`).  Constants are parameters of the specs, so that another design of this kind is another parser
(:mod:`kvmini.models.vodinex`, :mod:`kvmini.models.pipilix`, :mod:`kvmini.models.zipelix` and :mod:`kvmini.models.gebasun` are
four) and not another runner.

Weights are laid out for few, wide products.  Everything of a layer that reads the sublayer's input is one matrix
(``proj``: the branches' projections, the low-rank inputs of the delta rule and the residual gate), the two low-rank second
factors are one block-diagonal matrix (``low``), and the branches' output projections are one matrix over the concatenated
branch outputs (``out``; the branch scales are applied to the outputs before they are rounded, the bias is summed up front).
The key and value maps of latent attention exist per head, for single tokens that stay in the latent space (``absorb``: query
to latent, ``up``: latent to value), and as one matrix for prompts (``expand``: latent to all keys and values).  The input
dimension of every matrix is zero-padded to what the GEMM kernels take (:func:`pad_k`), activations likewise, so any size
runs on the same kernels.  How a matrix is stored is the :class:`Layout`'s business, which the ops provide."""

from __future__ import annotations

import math
from dataclasses import dataclass, field
from typing import Any, Callable, Dict, List, Optional, Tuple, Union

import torch

from .llama import interleave_gate_up


@dataclass(frozen=True)
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int = 0  # position i sees j <= i of its own chunk of this many positions (0: every j <= i)
    rot_base: float = 10000.0
    rot_dims: int = 0  # first dimensions of a head that are rotated (pairs i, i + rot_dims / 2)
    window: int = 0  # position i sees j with 0 <= i - j < window (0: every j <= i)
    keep: int = 0  # ... and the first ones of the sequence, j < keep
    gate: str = "head"  # the output gate: one per head, one per element of the concatenated heads ("element"), or "none"
    key_values: bool = False  # the values are the keys as projected, in front of norm and rotation
    norm_gains: bool = True  # the query / key norms have gains per dimension
    out_bias: bool = True
    sink: bool = False  # the softmax's denominator has one more term per head, exp of a learned number
    rel: bool = False  # a learned number per head and distance bucket is added to the scores (behind the scale)
    rel_max: int = 0  # the distance at which the last bucket is reached
    rel_buckets: int = 32  # (a checkpoint's come from its tensor, this is for random weights)

    @property
    def gates(self) -> int:
        return {"head": self.heads, "element": self.heads * self.vdim, "none": 0}[self.gate]


@dataclass(frozen=True)
class LatentSpec:
    """Softmax attention on latents: a token caches the normalised vector c (``kv_rank``), head h's key and value are W_uk[h] c and
    W_uv[h] c.  Positions: with ``rot_dim``, queries have as many more dimensions per head and a token one more key part of that
    size for all heads, both rotated (neighbouring dimensions 2i, 2i + 1 by position * rot_base^(-2i / rot_dim)); the part is cached
    behind the latent."""

    heads: int
    dim: int
    vdim: int
    kv_rank: int
    scale: float
    window: int = 0  # position i sees j with 0 <= i - j < window (0: every j <= i)
    rot_dim: int = 0
    rot_base: float = 10000.0
    gate: str = "head"  # the output gate: one per head, or one per element of the concatenated heads ("element")
    kv_from: int = -1  # the layer whose cache this one reads (-1: its own)

    kv_heads = 1  # one latent per token serves all heads

    @property
    def gates(self) -> int:
        return self.heads * self.vdim if self.gate == "element" else self.heads


@dataclass(frozen=True)
class DeltaSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int  # of the short convolutions
    decay_rank: int = 0  # ranks of the decay and output-gate projections: a checkpoint's come from its tensors, these are
    gate_rank: int = 0  # for random weights (0: dim)

    @property
    def channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim

    @property
    def state_shape(self) -> Tuple[int, int, int]:
        return self.heads, self.dim, self.vdim

    @property
    def ring_shape(self) -> Tuple[int, int]:
        return self.taps, self.channels


@dataclass(frozen=True)
class RetentionSpec:
    """Linear attention with a fixed decay per head, no softmax: S <- decay S + k v^T, o = S^T q; q and k rotated (pairs
    i, i + rot_dims / 2), k times dim^-1/2 behind it.  Each head's o is divided by its root mean square, the concatenated heads are
    gated with silu element by element."""

    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]
    rot_base: float = 10000.0
    rot_dims: int = 0

    ring_shape = None  # no convolution in front

    @property
    def kv_heads(self) -> int:
        return self.heads

    @property
    def state_shape(self) -> Tuple[int, int, int]:
        return self.heads, round_up(self.dim, 16), round_up(self.vdim, 16)  # (whole tiles of the matrix instructions)


@dataclass(frozen=True)
class StateSpaceSpec:
    """Linear attention whose decay and step size per head come from the token (state-space duality): with dt = softplus(dt + dt_bias),
    S <- exp(-exp(A) dt) S + dt b x^T (S is dim x vdim), o = S^T c + D x.  x (heads), b and c (groups of heads share them) come out of a
    short causal convolution with bias, silu behind it.  The concatenated heads are gated with silu element by element, then divided in
    ``norm_groups`` equal parts by their own root mean squares, with a gain per channel."""

    heads: int
    vdim: int
    dim: int  # rows of a head's state
    groups: int
    taps: int  # of the short convolution
    norm_groups: int = 1

    @property
    def kv_heads(self) -> int:
        return self.groups

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        return self.inner + 2 * self.groups * self.dim

    @property
    def state_shape(self) -> Tuple[int, int, int]:
        return self.heads, round_up(self.dim, 16), round_up(self.vdim, 16)  # (whole tiles of the matrix instructions)

    @property
    def ring_shape(self) -> Tuple[int, int]:
        return self.taps, self.channels


@dataclass(frozen=True)
class BranchSpec:
    mixer: Union[AttentionSpec, LatentSpec, DeltaSpec, RetentionSpec, StateSpaceSpec]
    tensors: str  # where the branch's tensors are, behind the layer's own prefix
    scale: float = 1.0


@dataclass(frozen=True)
class MoeSpec:
    """Mixture of experts: scores sigmoid(router), softmax(router) over all experts, or its softmax over the chosen ones alone
    ("chosen"); the ``top`` experts by score (plus a learned correction), weighted by their scores times ``scale``.  An expert, ``act``
    clamped: g = min(gate, limit), u = clamp(up, -limit, limit), g sigmoid(1.702 g) (u + 1) through ``down``; silu: silu(gate) up through
    ``down``; relu2: max(up, 0)^2 through ``down``, without a gate.  A shared expert (silu, or relu2 like the others, width
    ``shared_ff``) runs for every token, times the sigmoid of one more router row if ``shared_gate``."""

    experts: int
    top: int
    ff: int
    limit: float = math.inf
    scores: str = "sigmoid"
    scale: float = 1.0
    correction: bool = True
    act: str = "clamped"
    shared_ff: int = 0
    shared_gate: bool = True
    bias: bool = False  # the router has one, added to its logits

    @property
    def gated(self) -> bool:
        return self.act != "relu2"

    @property
    def glu(self) -> Tuple[float, float, float]:
        """(limit, a, b) of an expert's gate g sigmoid(a g) (u + b)."""
        return (self.limit, 1.702, 1.0) if self.act == "clamped" else (math.inf, 1.0, 0.0)


@dataclass(frozen=True)
class LayerSpec:
    branches: Tuple[BranchSpec, ...]
    ff: int = 0  # width of the gated MLP (0: the layer has none)
    act: str = "gelu_tanh"  # of the gate: gelu_tanh or silu
    moe: Optional[MoeSpec] = None  # instead of the MLP

    @property
    def feeds_forward(self) -> bool:
        return self.ff > 0 or self.moe is not None


@dataclass(frozen=True)
class LoopSpec:
    """Layers ``start`` .. ``stop`` - 1 run ``times`` times in a row, each pass with memory of its own.  Ahead of pass t the stream
    takes a vector of that pass (``loop.step``), and ahead of every pass but the first the embedding output once more."""

    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class LayerRun:
    layer: int
    begins: int = -1  # the pass that begins right ahead of this run (-1: none does)


@dataclass(frozen=True)
class HybridConfig:
    name: str
    vocab_size: int
    hidden_size: int
    layers: Tuple[LayerSpec, ...]
    rms_eps: float
    residual_mult: float = 1.0
    family: str = "hybrid"
    wiring: str = "gated"
    embed_scale: float = 1.0
    sine_positions: bool = False  # sines and cosines of position * 10000^(-2i / width), interleaved, are added to the embedding
    logit_scale: float = 1.0
    loop: Optional[LoopSpec] = None
    streams: int = 0  # of the hyper wiring
    tied_head: bool = False  # the LM head is the embedding table
    logit_softcap: float = 0.0  # c: logits become c tanh(logits / c) (0: they stay)
    max_position: int = 1 << 20
    bos_token_id: int = 1
    eos_token_id: int = -1  # none
    extra_eos_token_ids: Tuple[int, ...] = field(default=())

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @property
    def runs(self) -> Tuple[LayerRun, ...]:
        """The layers in the order they run."""
        lp = self.loop or LoopSpec(0, 0, 0)
        out = [LayerRun(i) for i in range(lp.start)]
        for t in range(lp.times):
            out += [LayerRun(i, t if i == lp.start else -1) for i in range(lp.start, lp.stop)]
        return tuple(out + [LayerRun(i) for i in range(lp.stop, len(self.layers))])

    @property
    def ld(self) -> int:
        """Elements per row of the residual stream."""
        return pad_k(self.hidden_size)

    @property
    def recurrent(self) -> bool:
        return any(isinstance(b.mixer, (DeltaSpec, RetentionSpec, StateSpaceSpec)) for la in self.layers for b in la.branches)


def pad_k(n: int) -> int:
    """Input widths the GEMM kernels take: 128 or a multiple of 256."""
    return 128 if n <= 128 else -(-n // 256) * 256


def round_up(n: int, m: int) -> int:
    return -(-n // m) * m


def check_config(cfg: HybridConfig) -> None:
    def bad(why: str) -> None:
        raise ValueError(f"{cfg.name}: {why}")

    if cfg.vocab_size < 1 or cfg.hidden_size < 1 or not cfg.layers:
        bad("vocabulary, width and layer list must not be empty")
    if cfg.wiring not in ("gated", "sandwich", "hyper", "parallel"):
        bad(f"unknown wiring {cfg.wiring!r}")
    if cfg.wiring == "hyper" and (not 1 <= cfg.streams <= 16 or cfg.loop is not None):
        bad(f"{cfg.streams} residual streams (1 to 16, in models without a loop)")
    if cfg.wiring == "parallel" and cfg.loop is not None:
        bad("a loop over layers of the parallel wiring")
    lp = cfg.loop
    if lp is not None and not (0 <= lp.start < lp.stop <= len(cfg.layers) and lp.times >= 1):
        bad(f"loop over layers {lp.start} .. {lp.stop}, {lp.times} times, of {len(cfg.layers)} layers")
    for i, la in enumerate(cfg.layers):
        if la.act not in ("gelu_tanh", "silu"):
            bad(f"layer {i}: unknown activation {la.act!r}")
        e = la.moe
        if e is not None and (e.scores not in ("sigmoid", "softmax", "chosen") or e.act not in ("clamped", "silu", "relu2") or e.shared_ff < 0):
            bad(f"layer {i}: scores {e.scores!r}, activation {e.act!r}, shared expert of width {e.shared_ff}")
        if e is not None and e.shared_ff and cfg.wiring not in ("hyper", "parallel"):
            bad(f"layer {i}: a shared expert in the {cfg.wiring} wiring")
        if cfg.wiring == "parallel" and la.ff:
            bad(f"layer {i}: a plain MLP in the parallel wiring")
        if e is not None and (la.ff or not 1 <= e.top <= min(e.experts, 64) or e.experts > 1024 or e.ff < 1):
            bad(f"layer {i}: {e.top} of {e.experts} experts of width {e.ff} (at most 64 of 1024)")
        for b in la.branches:
            m = b.mixer
            if m.heads < 1 or m.kv_heads < 1 or m.heads % m.kv_heads or m.dim < 1 or m.vdim < 1:
                bad(f"layer {i}: {m.heads} heads over {m.kv_heads} key heads of size {m.dim} / {m.vdim}")
            if isinstance(m, AttentionSpec) and (m.rot_dims % 2 or not 0 <= m.rot_dims <= m.dim or m.chunk < 0 or max(m.dim, m.vdim) > 1024):
                bad(f"layer {i}: rotated dimensions {m.rot_dims}, chunk {m.chunk}, head sizes {m.dim} / {m.vdim} (at most 1024)")
            if isinstance(m, AttentionSpec) and (m.window < 0 or m.keep < 0 or (m.chunk and (m.window or m.keep)) or (m.keep and not m.window) or m.gate not in ("head", "element", "none")):
                bad(f"layer {i}: window {m.window}, first tokens {m.keep}, chunk {m.chunk}, gate {m.gate!r}")
            if isinstance(m, AttentionSpec) and m.key_values and m.dim != m.vdim:
                bad(f"layer {i}: values of size {m.vdim} that are the keys of size {m.dim}")
            if isinstance(m, AttentionSpec) and m.rel and (m.chunk or m.rel_max < 1 or m.rel_buckets < 2):
                bad(f"layer {i}: a distance bias of {m.rel_buckets} buckets up to {m.rel_max}, chunk {m.chunk}")
            if isinstance(m, LatentSpec) and (m.kv_rank < 1 or m.window < 0 or max(m.dim, m.vdim, m.kv_rank) > 1024):
                bad(f"layer {i}: window {m.window}, latent size {m.kv_rank}, head sizes {m.dim} / {m.vdim} (at most 1024)")
            if isinstance(m, LatentSpec) and (m.rot_dim % 2 or not 0 <= m.rot_dim <= 512 or round_up(m.kv_rank, 4) + round_up(m.rot_dim, 4) > 1024 or m.gate not in ("head", "element")):
                bad(f"layer {i}: rotated part of {m.rot_dim} behind {m.kv_rank} (even, at most 512 and 1024 together), gate {m.gate!r}")
            if isinstance(m, LatentSpec) and m.kv_from >= 0:
                src = [x.mixer for x in cfg.layers[m.kv_from].branches] if m.kv_from < i else []
                if len(la.branches) != 1 or len(src) != 1 or not isinstance(src[0], LatentSpec) or src[0].kv_from >= 0 or \
                        (src[0].kv_rank, src[0].rot_dim, src[0].rot_base) != (m.kv_rank, m.rot_dim, m.rot_base):
                    bad(f"layer {i}: cannot read the latents of layer {m.kv_from} (an earlier one with its own, of the same sizes and rotation)")
            if isinstance(m, RetentionSpec) and (len(m.decay) != m.heads or not all(0 <= g <= 1 for g in m.decay) or m.rot_dims % 2 or not 0 <= m.rot_dims <= m.dim or max(m.dim, m.vdim) > 1024):
                bad(f"layer {i}: {len(m.decay)} decays of {m.heads} heads, rotated dimensions {m.rot_dims}, head sizes {m.dim} / {m.vdim} (at most 1024)")
            if isinstance(m, StateSpaceSpec) and (m.taps < 1 or m.norm_groups < 1 or m.inner % m.norm_groups):
                bad(f"layer {i}: {m.taps} convolution taps, {m.inner} channels in {m.norm_groups} parts")
            if isinstance(m, DeltaSpec) and (m.taps < 1 or m.dim > 512):
                bad(f"layer {i}: {m.taps} convolution taps, key size {m.dim} (at most 512)")


@dataclass
class AttentionWeights:
    q_off: int  # columns of the layer's projections
    k_off: int
    v_off: int
    g_off: int
    o_off: int  # column of the layer's concatenated branch outputs
    bias: torch.Tensor  # fp32, query | key | value
    q_norm: torch.Tensor
    k_norm: torch.Tensor
    sink: Optional[torch.Tensor] = None  # fp32 [heads]
    rel: Optional[torch.Tensor] = None  # fp32 [heads, distances]: what is added to a score at each distance (the last one: and beyond)


@dataclass
class LatentWeights:
    q_off: int  # columns of the layer's projections: queries, `dkp` per head
    c_off: int  # the latent before its norm, `rkp`
    g_off: int
    o_off: int  # column of the layer's concatenated branch outputs
    dkp: int  # padded sizes: query / key, value, latent
    dvp: int
    rkp: int
    c_norm: torch.Tensor  # fp32 [rkp], zero behind the true size
    absorb: Any  # per head: query -> latent space, [heads, rkp, dkp]
    up: Any  # per head: latent -> value, [heads, dvp, rkp]
    expand: Any = None  # latent -> every head's key, then every head's value, [heads dkp + heads dvp, rkp] (layouts with prompt kernels)
    r_off: int = 0  # the queries' rotated part, `rtp` per head
    rtp: int = 0
    kr_off: int = 0  # the rotated key part (in the cache it sits right behind the latent)


@dataclass
class MoeWeights:
    router: Any  # [experts, ld]
    correction: torch.Tensor  # fp32 [experts]
    gate_up: Any  # [experts, 2 ffp, ld], gate and up rows interleaved in eights (experts without a gate: [experts, ffp, ld])
    down: Any  # [experts, ld, ffp]
    ffp: int
    shared_gate_up: Any = None  # (the shared expert's gate is the router's last row)
    shared_down: Any = None
    bias: Optional[torch.Tensor] = None  # fp32 [experts], of the router


@dataclass
class RetentionWeights:
    q_off: int  # columns of the layer's projections
    k_off: int
    v_off: int
    g_off: int
    o_off: int  # column of the layer's concatenated branch outputs
    log2_decay: torch.Tensor  # fp32 [heads]


@dataclass
class StateSpaceWeights:
    z_off: int  # columns of the layer's projections: gates
    x_off: int  # the convolution's channels, x | b | c
    dt_off: int
    o_off: int  # column of the layer's concatenated branch outputs
    conv: torch.Tensor  # fp32 [taps, channels]
    conv_bias: torch.Tensor  # fp32, as the rest
    dt_bias: torch.Tensor
    a_log: torch.Tensor
    skip: torch.Tensor  # [heads]
    norm: torch.Tensor  # [inner]


BranchWeights = Union[AttentionWeights, LatentWeights, "DeltaWeights", RetentionWeights, StateSpaceWeights]


@dataclass
class HyperWeights:
    """One sublayer's weights over the streams, fp32."""

    read: torch.Tensor  # [streams]
    out: torch.Tensor  # [streams]
    mix: torch.Tensor  # [from, to]


@dataclass
class DeltaWeights:
    q_off: int
    k_off: int
    v_off: int
    b_off: int
    low_off: int  # low-rank inputs inside the projections, low_k columns
    low_k: int
    z_off: int  # decay inputs / output gates inside the low-rank product
    gate_off: int
    o_off: int
    low: Any  # weight: block-diagonal second factors
    conv: torch.Tensor  # fp32 [taps, channels]
    a_log: torch.Tensor
    dt_bias: torch.Tensor
    norm: torch.Tensor


@dataclass
class HybridLayer:
    proj: Any  # weight over the sublayer's input: branches, low-rank inputs, residual gate
    gate_off: int
    gate_bias: Optional[torch.Tensor]  # (None: no residual gate)
    norm: Optional[torch.Tensor]  # of the sublayer's result: one gain, or one per column (hyper, parallel: none)
    out: Any
    out_k: int
    out_gaps: bool  # the concatenated branch outputs have columns nobody writes
    out_bias: Optional[torch.Tensor]
    branches: List[BranchWeights]
    gate_up: Any = None
    down: Any = None
    gate2: Any = None
    gate2_bias: Optional[torch.Tensor] = None
    norm2: Optional[torch.Tensor] = None
    moe: Optional[MoeWeights] = None
    pre: Optional[torch.Tensor] = None  # sandwich, hyper, parallel: norms ahead of the two sublayers, fp32 [ld]
    pre2: Optional[torch.Tensor] = None
    hyper: Optional[HyperWeights] = None
    hyper2: Optional[HyperWeights] = None


@dataclass
class HybridWeights:
    cfg: HybridConfig
    embed: torch.Tensor  # [vocab, width]
    layers: List[HybridLayer]
    final_norm: torch.Tensor  # (times the logits' scale)
    lm_head: Any
    step: Optional[torch.Tensor] = None  # loop: fp32 [times, ld]
    tp_rank: int = 0
    tp_size: int = 1

    @property
    def device(self) -> torch.device:
        return self.embed.device


# ---- tensors of a checkpoint -------------------------------------------------------------------------------------
def branch_shapes(b: BranchSpec, width: int) -> Dict[str, Tuple[int, ...]]:
    m = b.mixer
    if isinstance(m, AttentionSpec):
        q, k, v = m.heads * m.dim, m.kv_heads * m.dim, m.kv_heads * m.vdim
        out: Dict[str, Tuple[int, ...]] = {"q": (q, width), "q.b": (q,), "k": (k, width), "k.b": (k,)}
        if not m.key_values:
            out.update({"v": (v, width), "v.b": (v,)})
        if m.norm_gains:
            out.update({"q.norm": (m.dim,), "k.norm": (m.dim,)})
        if m.sink:
            out["sink"] = (m.heads,)
        if m.rel:
            out["rel"] = (m.rel_buckets, m.heads)
        if m.gates:
            out["g"] = (m.gates, width)
        out["o"] = (width, m.heads * m.vdim)
        if m.out_bias:
            out["o.b"] = (width,)
        return out
    if isinstance(m, LatentSpec):
        own: Dict[str, Tuple[int, ...]] = {"dkv": (m.kv_rank + m.rot_dim, width), "dkv.norm": (m.kv_rank,)} if m.kv_from < 0 else {}
        return {"q": (m.heads * (m.dim + m.rot_dim), width), **own, "uk": (m.heads * m.dim, m.kv_rank), "uv": (m.heads * m.vdim, m.kv_rank), "g": (m.gates, width),
                "o": (width, m.heads * m.vdim)}
    if isinstance(m, RetentionSpec):
        qk, vs = (m.heads * m.dim, width), (m.heads * m.vdim, width)
        return {"q": qk, "k": qk, "v": vs, "g": vs, "o": vs[::-1]}
    if isinstance(m, StateSpaceSpec):
        return {"in": (m.inner + m.channels + m.heads, width), "conv": (m.channels, m.taps), "conv.b": (m.channels,), "dt_bias": (m.heads,), "A_log": (m.heads,), "D": (m.heads,),
                "norm": (m.inner,), "o": (width, m.inner)}
    q, v = m.kv_heads * m.dim, m.heads * m.vdim
    ra, rg = m.decay_rank or m.dim, m.gate_rank or m.dim
    return {"q": (q, width), "q.conv": (q, m.taps), "k": (q, width), "k.conv": (q, m.taps), "v": (v, width), "v.conv": (v, m.taps), "b": (m.heads, width), "A_log": (m.heads,), "norm": (m.vdim,),
            "a1": (ra, width), "a2": (m.heads * m.dim, ra), "dt_bias": (m.heads * m.dim,), "g1": (rg, width), "g2": (v, rg), "o": (width, v)}


def tensor_shapes(cfg: HybridConfig) -> Dict[str, Tuple[int, ...]]:
    w, gated = cfg.hidden_size, cfg.wiring == "gated"
    out: Dict[str, Tuple[int, ...]] = {"embed": (cfg.vocab_size, w)}
    if cfg.loop is not None:
        out["loop.step"] = (cfg.loop.times, w)

    def around(n: str, i: int) -> Dict[str, Tuple[int, ...]]:
        """Norms and gate of a layer's sublayer i, or its weights over the streams."""
        if cfg.wiring == "hyper":
            s = cfg.streams
            return {f"{n}norm{i}": (w,), f"{n}hc{i}.in": (s,), f"{n}hc{i}.out": (s,), f"{n}hc{i}.mix": (s, s)}
        if cfg.wiring == "parallel":
            return {f"{n}norm{i}": (w,)}
        return {f"{n}norm{i}": (), f"{n}rg{i}": (w, w), f"{n}rg{i}.b": (w,)} if gated else {f"{n}norm{i}": (w,), f"{n}norm{i}b": (w,)}

    for i, la in enumerate(cfg.layers):
        n = f"l{i}."
        out.update(around(n, 1))
        for b in la.branches:
            out.update({f"{n}{b.tensors}.{k}": s for k, s in branch_shapes(b, w).items()})
        if la.feeds_forward:
            out.update(around(n, 2))
        if la.ff:
            out.update({n + "mlp.gate": (la.ff, w), n + "mlp.up": (la.ff, w), n + "mlp.down": (w, la.ff)})
        if la.moe is not None:
            def ff(p: str, f: int, gated: bool) -> Dict[str, Tuple[int, ...]]:
                return {**({p + "gate": (f, w)} if gated else {}), p + "up": (f, w), p + "down": (w, f)}

            for e in range(la.moe.experts):
                out.update(ff(f"{n}mlp.e{e}.", la.moe.ff, la.moe.gated))
            out[n + "mlp.router"] = (la.moe.experts, w)
            if la.moe.bias:
                out[n + "mlp.router.b"] = (la.moe.experts,)
            if la.moe.correction:
                out[n + "mlp.correction"] = (la.moe.experts,)
            if la.moe.shared_ff:
                out.update(ff(n + "mlp.shared.", la.moe.shared_ff, la.moe.gated))
                if la.moe.shared_gate:
                    out[n + "mlp.shared.sg"] = (1, w)
    out["final.norm"] = () if gated else (w,)
    if not cfg.tied_head:
        out["head"] = (cfg.vocab_size, w)
    return out


RANKED = {"a1": 0, "a2": 1, "g1": 0, "g2": 1, "rel": 0}  # tensors with a free size, and where it is


def distance_buckets(buckets: int, longest: int, distances: int) -> List[int]:
    """Row of a table of distance biases for every distance below ``distances``: one row each below half of the ``buckets``, then rows for
    logarithmically wider ranges, the last one from ``longest`` on."""
    half = buckets / 2
    wide = math.log(longest / half) if longest > half else 0.0

    def row(n: int) -> int:
        if n < half:
            return n
        return buckets - 1 if wide == 0.0 or n >= longest else min(buckets - 1, int(half + math.floor(math.log(n / half) / wide * (buckets - half))))

    return [row(n) for n in range(distances)]


def random_tensors(cfg: HybridConfig, device: Any, dtype: torch.dtype, seed: int) -> Callable[[str], torch.Tensor]:
    """Random weights of a checkpoint's names and shapes, drawn when asked for (in order: layer by layer), so a large model
    never exists twice.  Matrices have variance 1 / fan-in; the rest is spread around its neutral value."""
    dev = torch.device(device)
    gen = torch.Generator(device=dev)
    gen.manual_seed(seed)
    shapes = tensor_shapes(cfg)

    def get(name: str) -> torch.Tensor:
        s = shapes[name]
        r = torch.randn(s, generator=gen, device=dev, dtype=torch.float32)
        leaf = name.rsplit(".", 1)[-1]
        if leaf.startswith("norm"):
            r = 1.0 + 0.1 * r
        elif leaf == "conv":
            r = r / math.sqrt(s[1])
        elif leaf in ("in", "out", "mix") and ".hc" in name:  # near one plain residual stream
            r = 0.1 * r + (1.0 / s[0] if leaf == "in" else 1.0 if leaf == "out" else torch.eye(s[0], device=dev))
        elif name == "embed" and cfg.tied_head:  # (logits of order one)
            r = r / math.sqrt(s[1])
        elif leaf == "correction":  # (small: choices spread evenly over the experts)
            r = 0.01 * r
        elif leaf in ("D", "sink", "rel"):
            pass
        elif leaf == "step" or (leaf == "b" and len(s) == 1):
            r = 0.1 * r
        elif leaf in ("A_log", "dt_bias"):
            r = r - 1.0
        elif name != "embed":
            r = r / math.sqrt(s[-1])
        return r.to(dtype)

    return get


# ---- packing -----------------------------------------------------------------------------------------------------
def _rows(parts: List[Tuple[int, torch.Tensor]], n: int, k: int, dtype: torch.dtype, device: Any) -> torch.Tensor:
    """Zero matrix [n, k] with the given blocks at (row, 0)."""
    w = torch.zeros((n, k), dtype=dtype, device=device)
    for off, p in parts:
        w[off : off + p.shape[0], : p.shape[1]] = p
    return w


def _vec(v: torch.Tensor, n: int) -> torch.Tensor:
    out = torch.zeros(n, dtype=torch.float32, device=v.device)
    out[: v.numel()] = v.float()
    return out


class Layout:
    """How matrices of a hybrid model are stored; this one keeps them row-major, at their own sizes.  Called with a matrix [out, in]:
    the form the engine's products take."""

    def __call__(self, w: torch.Tensor) -> Any:
        return w

    def out_rows(self, n: int) -> int:
        """Rows a stacked matrix of ``n`` rows takes."""
        return round_up(n, 64)

    def latent_pads(self, m: LatentSpec) -> Tuple[int, int, int]:
        """Padded query / key, value and latent sizes."""
        return m.dim, m.vdim, m.kv_rank

    def rot_pad(self, m: LatentSpec) -> int:
        """Padded size of the rotated part."""
        return m.rot_dim

    def expands(self, m: LatentSpec) -> bool:
        """Prompts run on expanded keys and values (else in the latent space, like single tokens)."""
        return False

    def heads(self, w: torch.Tensor, m: LatentSpec) -> Any:
        """Matrices [n, out, in], one per head of a latent branch."""
        return w

    def experts(self, w: torch.Tensor) -> Any:
        """Matrices [n, out, in], one per expert."""
        return w

    def expert_width(self, ff: int, gated: bool = True) -> int:
        return round_up(ff, 8)

    def router(self, w: torch.Tensor) -> Any:
        return w


def _head_blocks(w: torch.Tensor, heads: int, size: int, padded: int) -> torch.Tensor:
    """[heads * size, n] -> [heads * padded, n], zero rows behind every head's."""
    return w if size == padded else torch.nn.functional.pad(w.view(heads, size, -1), (0, 0, 0, padded - size)).reshape(heads * padded, -1)


def build_weights(cfg: HybridConfig, get: Callable[[str], torch.Tensor], dtype: torch.dtype, device: Any, layout: Layout) -> HybridWeights:
    """``get(name)``: a tensor of the checkpoint.  Layer by layer, so that at most one layer exists twice."""
    check_config(cfg)
    shapes = tensor_shapes(cfg)
    width, ld, gated = cfg.hidden_size, cfg.ld, cfg.wiring == "gated"

    def mat(name: str) -> torch.Tensor:
        t = get(name)
        want, leaf = shapes[name], name.rsplit(".", 1)[-1]
        if len(t.shape) != len(want) or any(a != b for d, (a, b) in enumerate(zip(t.shape, want)) if RANKED.get(leaf) != d):
            raise ValueError(f"{cfg.name}: tensor {name!r} has shape {tuple(t.shape)}, the configuration says {want}")
        return t.to(device=device, dtype=dtype)

    def vec(name: str) -> torch.Tensor:  # norms, biases and constants are kept in fp32
        t = get(name)
        if tuple(t.shape) != shapes[name]:
            raise ValueError(f"{cfg.name}: tensor {name!r} has shape {tuple(t.shape)}, the configuration says {shapes[name]}")
        return t.to(device=device, dtype=torch.float32).contiguous()

    def hyper(p: str) -> HyperWeights:
        return HyperWeights(vec(p + "in"), vec(p + "out"), vec(p + "mix"))

    def gain(name: str) -> torch.Tensor:
        return vec(name).view(1) if gated else _vec(vec(name), ld)

    def attention(m: AttentionSpec, p: str, section: Callable[..., int], o_off: int) -> AttentionWeights:
        q, k = section(mat(p + "q")), section(mat(p + "k"))
        v = k if m.key_values else section(mat(p + "v"))
        bias = torch.cat((vec(p + "q.b"), vec(p + "k.b"), vec(p + ("k.b" if m.key_values else "v.b"))))
        norms = [vec(p + n) if m.norm_gains else torch.ones(m.dim, device=device) for n in ("q.norm", "k.norm")]
        out = AttentionWeights(q, k, v, section(mat(p + "g")) if m.gates else 0, o_off, bias, *norms, vec(p + "sink") if m.sink else None)
        if m.rel:
            table = mat(p + "rel").float()
            n = max(m.rel_max, (table.shape[0] + 1) // 2) + 1  # (from there on every distance has the last row)
            n = min(m.window or n, n)
            out.rel = table[torch.tensor(distance_buckets(table.shape[0], m.rel_max, n), device=device)].T.contiguous()
        return out

    def latent(m: LatentSpec, p: str, section: Callable[..., int], o_off: int) -> LatentWeights:
        (dkp, dvp, rkp), rtp = layout.latent_pads(m), layout.rot_pad(m)
        wq = mat(p + "q").view(m.heads, m.dim + m.rot_dim, width)
        q, r, c, kr = section(_head_blocks(wq[:, : m.dim].reshape(-1, width), m.heads, m.dim, dkp)), 0, 0, 0
        if m.rot_dim:
            r = section(_head_blocks(wq[:, m.dim :].reshape(-1, width), m.heads, m.rot_dim, rtp))
        if m.kv_from < 0:
            dkv = mat(p + "dkv")
            c = section(torch.nn.functional.pad(dkv[: m.kv_rank], (0, 0, 0, rkp - m.kv_rank)))
            if m.rot_dim:
                kr = section(dkv[m.kv_rank :], rtp)
        g = section(mat(p + "g"))
        uk, uv = (_head_blocks(mat(p + n), m.heads, s, sp) for n, s, sp in (("uk", m.dim, dkp), ("uv", m.vdim, dvp)))
        uk, uv = (torch.nn.functional.pad(u, (0, rkp - m.kv_rank)) for u in (uk, uv))
        expand = layout(torch.cat((uk, uv)).contiguous()) if layout.expands(m) else None
        c_norm = _vec(vec(p + "dkv.norm"), rkp) if m.kv_from < 0 else torch.zeros(0, device=device)
        return LatentWeights(q, c, g, o_off, dkp, dvp, rkp, c_norm, layout.heads(uk.view(m.heads, dkp, rkp).transpose(1, 2).contiguous(), m),
                             layout.heads(uv.view(m.heads, dvp, rkp).contiguous(), m), expand, r, rtp, kr)

    def retention(m: RetentionSpec, p: str, section: Callable[..., int], o_off: int) -> RetentionWeights:
        q, k, v, g = (section(mat(p + n)) for n in "qkvg")
        log2 = [math.log2(x) if x > 0 else -1e4 for x in m.decay]  # (-1e4: no factor but the zeroth power's is above zero)
        return RetentionWeights(q, k, v, g, o_off, torch.tensor(log2, dtype=torch.float32, device=device))

    def state_space(m: StateSpaceSpec, p: str, section: Callable[..., int], o_off: int) -> StateSpaceWeights:
        z, xbc, dt = mat(p + "in").split((m.inner, m.channels, m.heads))
        return StateSpaceWeights(section(z), section(xbc), section(dt), o_off, mat(p + "conv").float().T.contiguous(), vec(p + "conv.b"), vec(p + "dt_bias"), vec(p + "A_log"), vec(p + "D"), vec(p + "norm"))

    def delta(m: DeltaSpec, p: str, section: Callable[..., int], o_off: int) -> DeltaWeights:
        q, k, v = section(mat(p + "q")), section(mat(p + "k")), section(mat(p + "v"))
        beta = section(mat(p + "b"))
        a1, a2, g1, g2 = mat(p + "a1"), mat(p + "a2"), mat(p + "g1"), mat(p + "g2")
        ra, rg = a1.shape[0], g1.shape[0]
        if a2.shape[1] != ra or g2.shape[1] != rg:
            raise ValueError(f"{cfg.name}: low-rank factors of {p} do not fit ({tuple(a1.shape)}, {tuple(a2.shape)}, {tuple(g1.shape)}, {tuple(g2.shape)})")
        low_k = pad_k(ra + rg)
        low_at = section(torch.cat((a1, g1)), low_k)
        gate_off = round_up(m.heads * m.dim, 8)
        low = torch.zeros((round_up(gate_off + m.heads * m.vdim, 64), low_k), dtype=dtype, device=device)
        low[: a2.shape[0], :ra] = a2
        low[gate_off : gate_off + g2.shape[0], ra : ra + rg] = g2
        conv = torch.cat((mat(p + "q.conv"), mat(p + "k.conv"), mat(p + "v.conv"))).float().T.contiguous()
        return DeltaWeights(q, k, v, beta, low_at, low_k, 0, gate_off, o_off, layout(low), conv, vec(p + "A_log"), vec(p + "dt_bias"), vec(p + "norm"))

    def experts(e: MoeSpec, p: str) -> MoeWeights:
        ffp = layout.expert_width(e.ff, e.gated)
        gate_up = torch.zeros((e.experts, 2 * ffp if e.gated else ffp, ld), dtype=dtype, device=device)
        down = torch.zeros((e.experts, ld, ffp), dtype=dtype, device=device)
        for i in range(e.experts):
            q = f"{p}e{i}."
            up = _rows([(0, mat(q + "up"))], ffp, ld, dtype, device)
            gate_up[i] = interleave_gate_up(_rows([(0, mat(q + "gate"))], ffp, ld, dtype, device), up) if e.gated else up
            down[i, :width, : e.ff] = mat(q + "down")
        router = [(0, mat(p + "router"))]
        out = MoeWeights(None, vec(p + "correction") if e.correction else torch.zeros(e.experts, device=device), layout.experts(gate_up), layout.experts(down), ffp)
        out.bias = vec(p + "router.b") if e.bias else None
        if e.shared_ff:
            if e.shared_gate:
                router.append((e.experts, mat(p + "shared.sg")))
            out.shared_gate_up, out.shared_down = mlp(e.shared_ff, p + "shared.", e.gated)
        out.router = layout.router(_rows(router, e.experts + len(router) - 1, ld, dtype, device))
        return out

    def mlp(ff: int, p: str, with_gate: bool = True) -> Tuple[Any, Any]:
        ffp = pad_k(ff)
        up = _rows([(0, mat(p + "up"))], ffp, ld, dtype, device)
        if with_gate:
            up = interleave_gate_up(_rows([(0, mat(p + "gate"))], ffp, ld, dtype, device), up).contiguous()
        return layout(up), layout(_rows([(0, mat(p + "down"))], ld, ffp, dtype, device))

    embed = mat("embed").contiguous()
    layers: List[HybridLayer] = []
    for li, la in enumerate(cfg.layers):
        n = f"l{li}."
        rows: List[Tuple[int, torch.Tensor]] = []
        off = 0

        def section(p: torch.Tensor, height: int = 0) -> int:
            nonlocal off
            at = off
            rows.append((at, p))
            off = round_up(at + (height or p.shape[0]), 8)
            return at

        outs: List[Tuple[int, torch.Tensor]] = []
        o_off, o_used, out_bias = 0, 0, None
        branches: List[BranchWeights] = []
        for b in la.branches:
            m, p = b.mixer, f"{n}{b.tensors}."
            pack_branch: Any = {AttentionSpec: attention, LatentSpec: latent, DeltaSpec: delta, RetentionSpec: retention, StateSpaceSpec: state_space}[type(m)]
            branches.append(pack_branch(m, p, section, o_off))
            if isinstance(m, AttentionSpec) and m.out_bias:
                ob = b.scale * _vec(vec(p + "o.b"), ld)
                out_bias = ob if out_bias is None else out_bias + ob
            o = mat(p + "o")
            outs.append((o_off, o))
            o_used = o_off + o.shape[1]
            o_off = round_up(o_used, 8)
        gate_off = section(mat(n + "rg1"), ld) if gated else 0
        proj = layout(_rows(rows, layout.out_rows(off), ld, dtype, device))
        out_k = pad_k(o_used)
        ow = torch.zeros((ld, out_k), dtype=dtype, device=device)
        for at, o in outs:
            ow[:width, at : at + o.shape[1]] = o
        layer = HybridLayer(proj, gate_off, _vec(vec(n + "rg1.b"), ld) if gated else None, gain(n + "norm1") if gated else gain(n + "norm1b") if cfg.wiring == "sandwich" else None, layout(ow), out_k,
                            sum(o.shape[1] for _, o in outs) != out_k, out_bias, branches)
        if not gated:
            layer.pre = gain(n + "norm1")
        if cfg.wiring == "hyper":
            layer.hyper = hyper(n + "hc1.")
        if la.feeds_forward:
            if cfg.wiring == "hyper":
                layer.hyper2 = hyper(n + "hc2.")
            elif cfg.wiring != "parallel":
                layer.norm2 = gain(n + ("norm2" if gated else "norm2b"))
            if gated:
                layer.gate2 = layout(_rows([(0, mat(n + "rg2"))], ld, ld, dtype, device))
                layer.gate2_bias = _vec(vec(n + "rg2.b"), ld)
            else:
                layer.pre2 = gain(n + "norm2")
        if la.ff:
            layer.gate_up, layer.down = mlp(la.ff, n + "mlp.")
        if la.moe is not None:
            layer.moe = experts(la.moe, n + "mlp.")
        layers.append(layer)
    final_norm = gain("final.norm") * cfg.logit_scale
    head = layout(_rows([(0, embed if cfg.tied_head else mat("head"))], cfg.vocab_size, ld, dtype, device))
    step = None
    if cfg.loop is not None:
        step = torch.nn.functional.pad(vec("loop.step"), (0, ld - width)).contiguous()
    return HybridWeights(cfg, embed, layers, final_norm, head, step)
