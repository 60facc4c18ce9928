"""Runner of hybrid decoders (:mod:`kvmini.models.hybrid`): the staging, graphs and stepping of :class:`ModelRunner` with
another forward pass and another kind of per-sequence memory.

Attention branches keep paged keys and values, latent branches paged latents (one pool of blocks for all layers, per-layer
sizes, one set of pages per run of a looped layer); recurrent branches keep a fixed-size state per sequence, indexed by the slot
the scheduler gives a running sequence (:class:`kvmini.engine.kv_cache.MixerMemory`).  A state is valid from the portion that starts at position 0 on, so slots need no
clearing when they change hands and a preempted sequence simply starts over.  What such a state rules out is checked here: a
prefix cannot be taken over from another request, and a step cannot be taken back (drafts to verify); models without a
recurrent branch have neither restriction.

Prompts of latent attention run on keys and values that are expanded, for the portions of the step and the earlier tokens their
windows reach, into a workspace (``spans``: which positions lie where).  The captured graph of a step shape holds a workspace as
large as the step itself, which is what prompts need that start at position 0; portions further in take a larger one
(:meth:`_step_variant`).

Where a layer's mixer and feed-forward read the same stream, the chosen experts run beside the mixer and the shared expert, on a
second HIP stream that is forked off and joined in every layer, in captured graphs as well.  What one stream allocates and the
other reads is held until the join, and the second stream starts every layer behind the first, so no memory is handed on early."""

from __future__ import annotations

from typing import Any, Callable, Dict, List, Optional, Tuple

import numpy as np
import torch

from kvmini.models.hybrid import AttentionSpec, DeltaSpec, HybridLayer, HybridWeights, LatentSpec, LayerRun, LayerSpec, RetentionSpec, StateSpaceSpec

from .kv_cache import MixerMemory
from .runner import ModelRunner, select_ops


class HybridRunner(ModelRunner):
    SPLIT_MAX_ROWS = 32
    QUERY_BLOCK = 32  # queries per work item of the prompt attention kernel
    LATENT_BLOCK = 128  # the same for latent attention
    CHUNK = 64  # tokens per work item of the retention and state-space kernels
    LATENT_SPLIT_MIN_CTX, LATENT_SPLIT_MAX_ROWS = 256, 64  # (all heads share a row's latents: there are few workgroups per row to begin with)

    # the residual stream behind every layer run: called on eager steps with (index of the run, stream)
    _after_layer: Optional[Callable[[int, torch.Tensor], None]] = None

    def _prepare_model(self, weights: HybridWeights) -> None:
        r = self.rcfg
        if self.tp_active or self.tp_size > 1:
            raise ValueError("tensor parallelism is not available for hybrid models")
        if r.quantization not in (None, "none"):
            raise ValueError(f"quantization {r.quantization!r} is not available for hybrid models")
        if r.kv_cache_dtype != "auto":
            raise ValueError(f"KV cache dtype {r.kv_cache_dtype!r} is not available for hybrid models")
        self.ops = select_ops(r.kernels, self.device)
        if hasattr(self.ops, "prepare_weights"):
            from kvmini.ops import hip_mixers as mixers
        else:
            from kvmini.ops import torch_mixers as mixers
        self.mixers = mixers
        self.dtype = weights.embed.dtype
        if hasattr(self.ops, "prepare_weights") and self.dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("hybrid models run in bf16 or fp32")
        # (fp32 products are the library's; only the engine's own kernels are captured into graphs)
        self.graphs_ok = self.dtype == torch.bfloat16
        self.nh = self.nkv = 1  # no kernel of the Llama path runs: its tile and split forms stay off
        self.hd = 0
        # the most keys any query of the model sees, and any query of a latent branch
        limit = self.rcfg.max_model_len
        mixers_ = [b.mixer for la in self.cfg.layers for b in la.branches]
        self.reach = max((min(m.window or limit, limit) for m in mixers_ if isinstance(m, LatentSpec)), default=0)
        self.longest = max([m.chunk or min(m.window + m.keep, limit) if m.chunk or m.window else limit for m in mixers_ if isinstance(m, AttentionSpec)] + [self.reach])
        self.expands = any(getattr(b, "expand", None) is not None for la in weights.layers for b in la.branches)
        self.retains = any(isinstance(m, (RetentionSpec, StateSpaceSpec)) for m in mixers_)
        self.aside = torch.cuda.Stream(self.device) if self.cfg.wiring == "parallel" and self.device.type == "cuda" and hasattr(mixers, "shared_expert") else None
        self.span_rows = 0  # rows of the expansion workspace the staged step needs
        self._rot: Dict[Tuple[float, int], Tuple[torch.Tensor, torch.Tensor]] = {}

    def _rotation(self, base: float, dims: int) -> Tuple[torch.Tensor, torch.Tensor]:
        """cos / sin of position * base^(-2i / dims), [positions, dims / 2]; shared by layers with the same constants."""
        key = (base, dims)
        if key not in self._rot:
            half = dims // 2
            inv = base ** (-2.0 * torch.arange(half, dtype=torch.float64) / max(1, dims))
            ang = torch.arange(self.rcfg.max_model_len, dtype=torch.float64)[:, None] * inv[None, :]
            self._rot[key] = (ang.cos().float().to(self.device), ang.sin().float().to(self.device))
        return self._rot[key]

    def _auto_num_blocks(self) -> int:
        r = self.rcfg
        want = r.max_num_seqs * self.max_blocks_per_seq + 64
        per_block = MixerMemory.block_bytes(self.cfg, self.block_size, self.dtype, self._pads)
        if self.device.type == "cuda" and per_block:
            free, _total = torch.cuda.mem_get_info(self.device)
            free -= MixerMemory.state_bytes(self.cfg, r.max_num_seqs, self.dtype, self._pads)
            return max(64, min(want, int(free * r.kv_memory_fraction) // per_block))
        return max(64, min(want, 4096))

    def _pads(self, m: Any) -> Tuple[int, ...]:
        return self.mixers.cache_pads(m, self.dtype, self.block_size)

    def _alloc_cache(self) -> None:
        self.kv_scale = None
        self.decode_layers = None
        self.memory = MixerMemory(self.cfg, self.num_blocks, self.block_size, self.rcfg.max_num_seqs, self.dtype, self.device, self._pads)
        # what a branch does, with its weights and memory: one callable (projections, outputs, staged step) per branch of every run
        self.branches: List[List[Callable[..., None]]] = []
        for run, mem in zip(self.cfg.runs, self.memory.runs):
            la, lw = self.cfg.layers[run.layer], self.w.layers[run.layer]
            self.branches.append([self._branch(b, bw, m) for b, bw, m in zip(la.branches, lw.branches, mem)])

    def _branch(self, b: Any, w: Any, mem: Tuple[Any, ...]) -> Callable[..., None]:
        mx, m, eps = self.mixers, b.mixer, self.cfg.rms_eps
        if isinstance(m, AttentionSpec):
            rot = self._rotation(m.rot_base, m.rot_dims)
            return lambda proj, mix, st: mx.attention(m, w, b.scale, eps, proj, mix, mem, rot, st)
        if isinstance(m, LatentSpec):
            turn = self._rotation(m.rot_base, m.rot_dim) if m.rot_dim else None
            return lambda proj, mix, st: mx.latent_attention(m, w, b.scale, eps, proj, mix, mem[0], st, turn)
        if isinstance(m, RetentionSpec):
            ret = mx.Retention(m, w, b.scale, eps, mem[0], self._rotation(m.rot_base, m.rot_dims))
            return lambda proj, mix, st: ret.run(proj, mix, st)
        if isinstance(m, StateSpaceSpec):
            space = mx.StateSpace(m, w, b.scale, eps, *mem)
            return lambda proj, mix, st: space.run(proj, mix, st)
        assert isinstance(m, DeltaSpec)
        delta = mx.DeltaState(m, w, b.scale, eps, *mem)
        return lambda proj, mix, st: delta.run(proj, self.ops.linear(proj[:, w.low_off : w.low_off + w.low_k], w.low), mix, st)

    def set_spec_width(self, width: int) -> None:
        if width > 1 and self.cfg.recurrent:
            raise ValueError("speculative decoding is not available for models with a recurrent state: a rejected draft cannot be taken back")
        super().set_spec_width(width)

    # ---- staging ---------------------------------------------------------------------------------------------------
    def _extra_staging(self) -> List[Tuple[str, int]]:
        smax = self.rcfg.max_num_seqs
        self.max_query_blocks = self.tmax // self.QUERY_BLOCK + smax
        self.max_latent_blocks = self.tmax // self.LATENT_BLOCK + smax
        spans = [("spans", 3 * smax), ("latent_blocks", 4 * self.max_latent_blocks)] if self.expands else []
        if self.retains:
            self.max_chunks = self.tmax // self.CHUNK + smax
            spans += [("chunks", 4 * self.max_chunks), ("first_chunk", smax)]
        return spans + [("tok_kind", self.tmax), ("tok_off", self.tmax), ("singles", smax), ("portions", 5 * smax), ("query_blocks", 4 * self.max_query_blocks)]

    def _stage_portions(self, st: np.ndarray, portions: List[Tuple[int, int, int, int]], t: int, t_pad: int) -> None:
        o_k, o_o, o_s, o_p, o_b = (self._off[k][0] for k in ("tok_kind", "tok_off", "singles", "portions", "query_blocks"))
        smax, mb = self.rcfg.max_num_seqs, self.max_query_blocks
        pa = st[o_p : o_p + 5 * smax].reshape(5, smax)
        ba = st[o_b : o_b + 4 * mb].reshape(4, mb)
        pa[1] = 0
        ba[1] = 0
        nb = ns = nt = 0  # query blocks, single rows, tiles (staged by the caller, in this order)
        for j, (row, n, pos, slot) in enumerate(portions):
            pa[:, j] = (row, n, pos, slot, nt)
            st[o_k + row : o_k + row + n] = 1 if n == 1 else 2
            st[o_o + row : o_o + row + n] = np.arange(n, dtype=np.int32)
            if n == 1:
                st[o_s + ns] = row
                ns += 1
            else:
                nt += (n + 15) // 16
                for off in range(0, n, self.QUERY_BLOCK):
                    ba[:, nb] = (row + off, min(self.QUERY_BLOCK, n - off), pos + off, slot)
                    nb += 1
        if self.expands:
            self._stage_spans(st, portions)
        if self.retains:
            self._stage_chunks(st, portions)
        st[o_s + ns : o_s + smax] = -1
        st[o_k + t : o_k + t_pad] = 0
        st[o_o + t : o_o + t_pad] = 0

    def _stage_spans(self, st: np.ndarray, portions: List[Tuple[int, int, int, int]]) -> None:
        """Where the keys of the step's prompt portions lie in the expansion workspace, and its query blocks."""
        smax, mb = self.rcfg.max_num_seqs, self.max_latent_blocks
        o_p, o_b = self._off["spans"][0], self._off["latent_blocks"][0]
        pa, ba = st[o_p : o_p + 3 * smax].reshape(3, smax), st[o_b : o_b + 4 * mb].reshape(4, mb)
        pa[:], ba[1] = 0, 0
        at = nb = 0
        for row, n, pos, slot in portions:
            if n == 1:
                continue
            first = max(0, pos - self.reach + 1)
            pa[:, slot] = (at, first, pos + n - first)  # first row, first position, rows
            for off in range(0, n, self.LATENT_BLOCK):
                ba[:, nb] = (row + off, min(self.LATENT_BLOCK, n - off), pos + off, at - first)  # (the workspace row of position p is the last number + p)
                nb += 1
            at += pos + n - first
        self.span_rows = at

    def _stage_chunks(self, st: np.ndarray, portions: List[Tuple[int, int, int, int]]) -> None:
        """The work items of retention and state spaces: pieces of the portions of several tokens, and each portion's first one."""
        o_c, o_f, mc = self._off["chunks"][0], self._off["first_chunk"][0], self.max_chunks
        ca = st[o_c : o_c + 4 * mc].reshape(4, mc)
        ca[1] = 0
        nc = 0
        for j, (row, n, pos, slot) in enumerate(portions):
            st[o_f + j] = nc
            if n > 1:
                for off in range(0, n, self.CHUNK):
                    ca[:, nc] = (row + off, min(self.CHUNK, n - off), pos + off, slot)
                    nc += 1

    def _step_variant(self, t_pad: int, decode_only: int) -> int:
        """Rows of the expansion workspace when the step needs more than its graph's (a power of two: few shapes)."""
        return 1 << (self.span_rows - 1).bit_length() if self.expands and not decode_only and self.span_rows > t_pad else 0

    def step_kind(self, t_pad: int, decode_only: bool, max_ctx: int) -> int:
        """0: portions of several tokens, 1: decoding, 2: decoding with some long context, few rows (shared out over workgroups)."""
        if not decode_only:
            return 0
        ctx, rows = (self.LATENT_SPLIT_MIN_CTX, self.LATENT_SPLIT_MAX_ROWS) if self.reach else (self.SPLIT_KV_MIN_CTX, self.SPLIT_MAX_ROWS)
        return 2 if min(max_ctx, self.longest) >= ctx and t_pad <= rows else 1

    def capture_graphs(self, buckets: Any = None) -> None:
        if self.graphs_ok:
            super().capture_graphs(buckets)

    # ---- forward ---------------------------------------------------------------------------------------------------
    def forward(self, t_pad: int, max_blocks: Optional[int] = None, decode_only: int = 0, quads: bool = False, dec_split: int = 0, pf_split: int = 0) -> torch.Tensor:
        ops, mx, cfg, w = self.ops, self.mixers, self.cfg, self.w
        smax = self.rcfg.max_num_seqs
        few = min(smax, t_pad)
        n_blocks = min(self.max_query_blocks, t_pad // self.QUERY_BLOCK + few)
        n_tiles = min(self.max_tiles, t_pad // 16 + min(smax, t_pad // 2))
        st = mx.Step(*(self._dev(k, t_pad) for k in ("tokens", "positions", "slots", "tok_seq", "tok_kind", "tok_off")), self._dev("block_tables").view(smax, self.max_blocks_per_seq),
                     self._dev("singles", few), self._dev("portions").view(5, smax), self._dev("query_blocks").view(4, self.max_query_blocks), n_blocks,
                     self._dev("tiles").view(4, self.max_tiles), n_tiles, bool(decode_only), decode_only == 2)
        if self.expands and not decode_only:
            st.spans, st.latent_blocks = self._dev("spans").view(3, smax), self._dev("latent_blocks").view(4, self.max_latent_blocks)
            st.n_latent_blocks = min(self.max_latent_blocks, t_pad // self.LATENT_BLOCK + min(smax, t_pad // 2))
            st.span_rows = pf_split or t_pad
        if self.retains and not decode_only:
            st.chunks, st.first_chunk = self._dev("chunks").view(4, self.max_chunks), self._dev("first_chunk")
            st.n_chunks = min(self.max_chunks, t_pad // self.CHUNK + min(smax, t_pad // 2))
        runs, gated, hyper, parallel, dt, width, eps = cfg.runs, cfg.wiring == "gated", cfg.wiring == "hyper", cfg.wiring == "parallel", self.dtype, cfg.hidden_size, cfg.rms_eps
        again = cfg.loop is not None and cfg.loop.times > 1  # the embedding output is added to the stream later on
        x, xb, start = mx.embed_stream(w.embed, st.tokens, self._dev("feed", t_pad), self.out_ids, cfg.ld, cfg.embed_scale, st.positions if cfg.sine_positions else None, again)

        def join(run: LayerRun) -> Any:
            """What the stream takes ahead of a run: (rows or None, vector)."""
            return None if run.begins < 0 else (start if run.begins > 0 else None, w.step[run.begins])

        if hyper:  # x becomes the streams [T, streams, ld]
            x, xb = mx.split_streams(x, cfg.streams, w.layers[runs[0].layer].hyper.read, w.layers[runs[0].layer].pre, eps, width, dt)
        elif parallel:  # xb, xb2: the inputs of a layer's mixer and feed-forward
            first = w.layers[runs[0].layer]
            xb, xb2 = mx.parallel_residual(x, None, None, None, first.pre, first.pre2, eps, width, dt)
        elif not gated:
            xb = mx.stream_norm(x, join(runs[0]), w.layers[runs[0].layer].pre, eps, width, dt)
        observed = self._after_layer is not None
        for ri, run in enumerate(runs):
            la, lw = cfg.layers[run.layer], w.layers[run.layer]
            # behind the run: the norm its successor's input takes (gated: only the head's does) and what the stream takes first
            ahead = runs[ri + 1] if ri + 1 < len(runs) else None
            fin = w.final_norm if ahead is None else None if gated else w.layers[ahead.layer].pre
            jn = None if ahead is None else join(ahead)
            if parallel and la.feeds_forward and self.aside is not None:
                main = torch.cuda.current_stream(self.device)
                self.aside.wait_stream(main)
                with torch.cuda.stream(self.aside):
                    chosen = mx.experts(la.moe, lw.moe, xb2, st, shared=False)
            proj = ops.linear(xb, lw.proj)
            mix = (torch.zeros if lw.out_gaps else torch.empty)((t_pad, lw.out_k), dtype=dt, device=self.device)
            for branch in self.branches[ri]:
                branch(proj, mix, st)
            last = not la.feeds_forward
            if parallel:
                y, y2 = ops.linear(mix, lw.out, allow_slabs=True), None
                if not last and self.aside is None:
                    y2 = self._feed_forward(la, lw, xb2, st)
                elif not last:
                    y2 = mx.with_shared(chosen, la.moe, lw.moe, xb2)
                    main.wait_stream(self.aside)
                xb, xb2 = mx.parallel_residual(x, y, lw.out_bias, y2, fin, None if ahead is None else w.layers[ahead.layer].pre2, eps, width, dt)
                if observed:
                    self._after_layer(ri, x)
                continue
            if hyper:
                done = (mx.all_streams(cfg.streams, self.device), fin) if ahead is None else (w.layers[ahead.layer].hyper.read, fin)
                xb = mx.hyper_residual(x, ops.linear(mix, lw.out, allow_slabs=True), lw.hyper, *(done if last else (lw.hyper2.read, lw.pre2)), eps, width, dt)
                if not last:
                    xb = mx.hyper_residual(x, self._feed_forward(la, lw, xb, st), lw.hyper2, *done, eps, width, dt)
                if observed:
                    self._after_layer(ri, x.sum(1))
                continue
            gate = proj[:, lw.gate_off : lw.gate_off + cfg.ld] if gated else None
            xb = mx.gated_residual(x, ops.linear(mix, lw.out, allow_slabs=True), lw.out_bias, gate, lw.gate_bias, lw.norm, cfg.residual_mult, eps, width, dt,
                                   lw.pre2 if not last else None if observed else fin, jn if last and not observed else None)
            if not last:
                if gated:
                    gate = ops.linear(xb, lw.gate2, allow_slabs=True)
                xb = mx.gated_residual(x, self._feed_forward(la, lw, xb, st), None, gate, lw.gate2_bias, lw.norm2, cfg.residual_mult, eps, width, dt, None if observed else fin, None if observed else jn)
            if observed:
                self._after_layer(ri, x)
                xb = mx.stream_norm(x, jn, fin, eps, width, dt)
        hs = torch.index_select(xb, 0, self._dev("sample_idx", t_pad)[: self.sample_rows(t_pad)])
        logits = ops.linear(hs, w.lm_head)
        if cfg.logit_softcap:
            mx.softcap(logits, cfg.logit_softcap)
        self.out_ids[: logits.shape[0]].copy_(ops.greedy_sample(logits))
        return logits

    def _feed_forward(self, la: LayerSpec, lw: HybridLayer, xb: torch.Tensor, st: Any) -> Any:
        if lw.moe is not None:
            return self.mixers.experts(la.moe, lw.moe, xb, st)
        return self.ops.linear((self.ops.linear_swiglu if la.act == "silu" else self.ops.linear_geglu)(xb, lw.gate_up), lw.down, allow_slabs=True)
