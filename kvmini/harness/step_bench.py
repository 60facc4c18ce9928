"""Device time of prefill and decode steps of the hybrid decoders beside a Llama decoder of equal width, MLP and depth
(``bench.py --workload steps``): random weights, a few layers at real sizes, the engine's own graphs replayed on staged steps.

Per size and step shape the line holds milliseconds per step, tokens per second, and how far the step is from its floor:
the larger of the weight bytes (plus K / V, latents and recurrent state of the step's sequences, read and written) over the HBM
rate and the matrix work over the bf16 MFMA rate.  Of a mixture of experts the floor counts the matrices that evenly spread choices
would touch."""

from __future__ import annotations

import time
from typing import Any, Dict, List, Tuple

import torch

HBM_BYTES_PER_S = 8.0e12
MFMA_FLOPS = 2.5e15

# width, MLP, heads, kv heads, head size, delta heads, delta key heads, delta key / value size, pattern, vocabulary
SIZES: Dict[str, Tuple[Any, ...]] = {
    "1b-layers": (2048, 8192, 32, 8, 64, 16, 16, 128, 128, "PPDP", 32768),
    "8b-layers": (4096, 14336, 32, 8, 128, 32, 32, 128, 128, "PPDP", 32768),
}
CHUNK = 8192
# Pipilix layers of the same width and MLP: heads, head size, value size, latent size, window, experts, chosen, expert width, pattern
PIPILIX: Dict[str, Tuple[Any, ...]] = {
    "1b-layers": (16, 128, 128, 512, 4096, 64, 6, 1408, "DMMM"),
    "8b-layers": (32, 128, 128, 512, 4096, 64, 6, 2304, "DMMM"),
}
# Zipelix layers: as Pipilix's with a rotated part instead of the window; retention heads, sizes; shared expert's width; pattern
ZIPELIX: Dict[str, Tuple[Any, ...]] = {
    "1b-layers": (16, 128, 64, 128, 512, 16, 128, 128, 64, 6, 1408, 2816, "LDRMSMRM"),
    "8b-layers": (32, 128, 64, 128, 512, 32, 128, 128, 64, 6, 2304, 4608, "LDRMSMRM"),
}
# Gebasun layers of the same width: heads, kv heads, head size, window, kept first tokens, rotated dimensions; state-space heads, head size, rows
# of the state, groups; experts, chosen, expert width, shared expert's width; pattern
GEBASUN: Dict[str, Tuple[Any, ...]] = {
    "1b-layers": (32, 8, 64, 4096, 64, 32, 64, 64, 128, 1, 64, 6, 1408, 2816, "BMSMAMSM"),
    "8b-layers": (32, 8, 128, 4096, 64, 64, 128, 64, 128, 1, 64, 6, 2304, 4608, "BMSMAMSM"),
}
DESIGNS = ("vodinex", "pipilix", "zipelix", "gebasun", "llama")


def configs(size: str) -> Tuple[Any, ...]:
    from kvmini.models import gebasun, pipilix, zipelix
    from kvmini.models.llama import LlamaConfig
    from kvmini.models.vodinex import stack

    width, ff, nh, nkv, hd, dh, dk, ddim, dv, pattern, vocab = SIZES[size]
    hy = stack(f"vodinex-{size}", vocab, width, ff, pattern, nh, nkv, hd, hd, CHUNK, dh, dk, ddim, dv, ranks=128, mult=0.5)
    ll = LlamaConfig(f"llama-{size}", vocab, width, ff, len(pattern), nh, nkv, hd, 500000.0, 1e-5, 8192, 1, 2)
    ph, pd, pv, rank, window, experts, top, eff, pat = PIPILIX[size]
    pp = pipilix.stack(f"pipilix-{size}", vocab, width, pat, ph, pd, pv, rank, window, ff, experts, top, eff, embed_scale=16.0)
    zh, zd, zr, zv, rank, rh, rd, rv, experts, top, eff, shared, pat = ZIPELIX[size]
    zp = zipelix.stack(f"zipelix-{size}", vocab, width, pat, zh, zd, zr, zv, rank, rh, rd, rv, ff, experts, top, eff, shared)
    *sizes, pat = GEBASUN[size]
    return hy, pp, zp, gebasun.stack(f"gebasun-{size}", vocab, width, pat, *sizes), ll


def matrix_elements(w: Any) -> int:
    """Elements of the matrices a step streams (the LM head included, the embedding table not)."""
    n = w.lm_head.numel()
    for la in w.layers:
        for v in list(vars(la).values()) + [getattr(b, "low", None) for b in getattr(la, "branches", [])]:
            if hasattr(v, "numel") and hasattr(v, "shape") and len(v.shape) == 2:
                n += v.numel()
    return n


def mixed_floor(cfg: Any, rows: int, seqs: int, ctx: int) -> Tuple[float, float]:
    """(bytes, matrix work) of a step of a model whose layers have one mixer each and, maybe, experts, embedding and head left out."""
    from kvmini.models.hybrid import AttentionSpec, RetentionSpec, StateSpaceSpec

    mem = flops = 0.0
    w = cfg.hidden_size
    for la in cfg.layers:
        m = la.branches[0].mixer
        if isinstance(m, StateSpaceSpec):
            params = w * (m.inner + m.channels + m.heads + m.inner)
            mem += 2.0 * params + 8.0 * seqs * m.inner * m.dim
            flops += 2.0 * rows * params + 4.0 * rows * m.inner * m.dim
        elif isinstance(m, AttentionSpec):
            params = w * (2 * m.heads * m.dim + m.kv_heads * m.dim + m.gates)
            seen, row = min(ctx, m.window or ctx), m.dim + (m.rot_dims if m.key_values else m.vdim)  # (one row can be key and value)
            mem += 2.0 * params + 2.0 * (seqs * seen if seqs == rows else rows) * m.kv_heads * row
            flops += 2.0 * rows * params + 2.0 * rows * (seen if seqs == rows or ctx > (m.window or ctx) else seen / 2) * m.heads * (m.dim + m.vdim)
        elif isinstance(m, RetentionSpec):
            params = w * m.heads * (2 * m.dim + 3 * m.vdim)
            mem += 2.0 * params + 8.0 * seqs * m.heads * m.dim * m.vdim
            flops += 2.0 * rows * params + 4.0 * rows * m.heads * m.dim * m.vdim
        else:
            hd, row = m.heads * (m.dim + m.vdim), m.kv_rank + m.rot_dim
            params = w * (m.heads * (m.dim + m.rot_dim) + (row if m.kv_from < 0 else 0) + m.gates + m.heads * m.vdim) + m.kv_rank * hd
            mem += 2.0 * params
            flops += 2.0 * rows * params
            seen = min(ctx, m.window or ctx)
            if seqs == rows:  # single tokens: in the latent space
                mem += 2.0 * seqs * seen * row
                flops += 2.0 * rows * seen * m.heads * (row + m.kv_rank)
            else:  # prompts from position 0: on expanded keys and values
                mem += 2.0 * rows * row
                flops += 2.0 * rows * (seen / 2 if ctx <= (m.window or ctx) else seen) * (hd + m.heads * m.rot_dim)
        if la.ff:
            mem += 6.0 * w * la.ff
            flops += 6.0 * rows * w * la.ff
        if la.moe is not None:
            e = la.moe
            touched = e.experts * (1.0 - (1.0 - e.top / e.experts) ** rows)
            matrices = 3 if e.gated else 2
            mem += 2.0 * (w * e.experts + matrices * w * (touched * e.ff + e.shared_ff))
            flops += 2.0 * rows * w * (e.experts + matrices * (e.top * e.ff + e.shared_ff))
    return mem, flops


def step_floor_ms(eng: Any, rows: int, head_rows: int, seqs: int, ctx: int) -> float:
    cfg, head = eng.mcfg, eng.weights.lm_head.numel()
    if getattr(cfg, "wiring", "") in ("sandwich", "hyper", "parallel"):
        mem, flops = mixed_floor(cfg, rows, seqs, ctx)
        return max((mem + 2.0 * head) / HBM_BYTES_PER_S, (flops + 2.0 * head * head_rows) / MFMA_FLOPS) * 1e3
    n = matrix_elements(eng.weights)
    mem, flops = 2.0 * n, 2.0 * (n - head) * rows + 2.0 * head * head_rows
    if hasattr(cfg, "recurrent"):
        from kvmini.models.hybrid import AttentionSpec

        for la in cfg.layers:
            for b in la.branches:
                m = b.mixer
                if isinstance(m, AttentionSpec):
                    mem += 2.0 * seqs * ctx * m.kv_heads * (m.dim + m.vdim)
                    flops += 2.0 * rows * (ctx if seqs == rows else ctx / 2) * m.heads * (m.dim + m.vdim)
                else:
                    mem += 8.0 * seqs * m.heads * m.dim * m.vdim
                    flops += 6.0 * rows * m.heads * m.dim * m.vdim
    else:
        mem += 4.0 * cfg.num_layers * seqs * ctx * cfg.kv_size
        flops += 4.0 * cfg.num_layers * rows * (ctx if seqs == rows else ctx / 2) * cfg.q_size
    return max(mem / HBM_BYTES_PER_S, flops / MFMA_FLOPS) * 1e3


def time_step(eng: Any, portions: List[Tuple[int, int]], iters: int) -> float:
    """Milliseconds of the step that brings ``tokens`` more tokens to sequences that hold ``start`` already (their contents do not
    matter for time): staged once, its graph replayed."""
    from kvmini.engine.scheduler import Batch, ScheduledChunk

    r, sch = eng.runner, eng.scheduler
    chunks = []
    for j, (start, n) in enumerate(portions):
        s = eng.make_sequence([(7 * i + 131 * j) % 1000 + 3 for i in range(start + n)])
        s.slot = sch._free_slots.pop()
        s.blocks = eng.bm.allocate(-(-(start + n) // eng.bm.block_size))
        chunks.append(ScheduledChunk(s, start, n, True))
    batch = Batch(chunks, sum(c.n_tokens for c in chunks))
    with torch.no_grad():
        h = r.launch(batch)
        r.collect(h)
        key, max_ctx = h.key, max(c.start + c.n_tokens for c in chunks)
        run = lambda: r._run_staged(key[0], max_ctx, key[1])  # noqa: E731
        for _ in range(3):
            run()
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        for _ in range(iters):
            run()
        torch.cuda.synchronize()
    ms = (time.perf_counter() - t0) * 1e3 / iters
    for c in chunks:
        eng.bm.free(c.seq.blocks)
        sch._free_slots.append(c.seq.slot)
    return ms


def run(sizes: List[str], iters: int, prompt: int = 2048, ctx: int = 1024, batches: Tuple[int, ...] = (1, 16, 64), only: str = "") -> Dict[str, Any]:
    from kvmini.engine.engine import EngineConfig, LLMEngine
    from kvmini.models.registry import random_weights

    out: Dict[str, Any] = {}
    for size in sizes:
        for kind, cfg in zip(DESIGNS, configs(size)):
            if only and kind != only:
                continue
            w = random_weights(cfg, "cuda:0", torch.bfloat16, seed=1)
            eng = LLMEngine(EngineConfig(model=cfg.name, device="cuda:0", max_num_seqs=64, max_batched_tokens=prompt, max_model_len=max(prompt, ctx + 64) + 64, num_blocks=64 * (ctx // 16 + 8) + prompt // 16),
                            weights=w)
            eng.warmup()
            res: Dict[str, Any] = {} if kind in ("pipilix", "zipelix", "gebasun") else {"matrix_elements_M": round(matrix_elements(eng.weights) / 1e6, 1)}
            cases = [(f"prefill_{prompt}", [(0, prompt)]), (f"prefill_4x{prompt // 4}", [(0, prompt // 4)] * 4)] + [(f"decode_{b}", [(ctx, 1)] * b) for b in batches]
            for name, portions in cases:
                ms = time_step(eng, portions, iters)
                rows = sum(n for _, n in portions)
                head_rows = eng.runner.sample_rows(eng.runner.bucket_for(rows))
                floor = step_floor_ms(eng, rows, head_rows, len(portions), max(s + n for s, n in portions))
                res[name] = {"ms": round(ms, 4), "tokens_per_s": round(rows / ms * 1e3, 1), "floor_ms": round(floor, 4), "times_floor": round(ms / floor, 2)}
            out.setdefault(size, {})[kind] = res
            del eng, w
            torch.cuda.empty_cache()
    return out
