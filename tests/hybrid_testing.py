"""Shared by the tests of hybrid decoder designs: back ends, checkpoints, staged steps, feeding of requests, comparison."""

import json
import os

import pytest
import torch

from kvmini.engine.replay import Replay, engine_for

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BACKENDS = [pytest.param(("cpu", "fp32"), id="cpu"), pytest.param(("cuda:0", "fp32"), id="hip-fp32", marks=pytest.mark.gpu), pytest.param(("cuda:0", "bf16"), id="hip-bf16", marks=pytest.mark.gpu)]
TYPES = {"fp32": torch.float32, "bf16": torch.bfloat16}


def mixers_of(device):
    if device == "cpu":
        from kvmini.ops import torch_mixers as m
    else:
        from kvmini.ops import hip_mixers as m
    return m


def save(path, doc, w):
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(doc, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in w.items()}, os.path.join(path, "model.safetensors"))
    return str(path)


def tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def close(got, want, dtype, what=""):
    """Row by row: rms of the difference over the vocabulary against the spread of the logits."""
    d = got.double() - want
    err = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.std(-1).mean()
    lim = 2e-5 if dtype == "fp32" else 0.05
    assert torch.isfinite(got).all() and float(err.max()) < lim, (what, float(err.max()), int(err.argmax()))


def feed(rp, plan, reqs, end=()):
    """Run steps of [(id, tokens)] asking for every logit; returns id -> logits rows in order."""
    at, out = {}, {}
    for step in plan:
        ents = []
        for i, n in step:
            lo = at.get(i, 0)
            ents.append({"id": i, "tokens": reqs[i][lo : lo + n], "want": list(range(n))})
            at[i] = lo + n
        lg = rp.step(ents, [i for i, _ in step if at[i] == len(reqs[i])])
        r = 0
        for i, n in step:
            out.setdefault(i, []).append(lg[r : r + n])
            r += n
    return {i: torch.cat(v) for i, v in out.items()}


def make_step(mx, portions, device, block_size=16, n_blocks=64, seed=0, long=False, reach=0, per=16):
    """Staged arrays of a step: portions = [(tokens, first position, slot)], pages in shuffled order.  ``reach``: the most keys a query of
    a latent branch sees (the workspace then holds what the portions see, the first portion's rows last)."""
    smax = 1 + max(s for _, _, s in portions)
    perm = (torch.randperm(n_blocks - 1, generator=torch.Generator().manual_seed(seed)) + 1)[: smax * per].view(smax, per)
    pos, seq, kind, off, seg, blk, slot, one, tile, chunk, first_chunk = [], [], [], [], [], [], [], [], [], [], []
    for n, p0, s in portions:
        seg.append((len(pos), n, p0, s, len(tile)))
        first_chunk.append(len(chunk))
        if n > 1:
            chunk += [(len(pos) + o, min(64, n - o), p0 + o, s) for o in range(0, n, 64)]
        if n == 1:
            one.append(len(pos))
        else:
            tile += [(len(pos) + o, min(16, n - o), p0 + o, s) for o in range(0, n, 16)]
            blk += [(len(pos) + o, min(32, n - o), p0 + o, s) for o in range(0, n, 32)]
        for i in range(n):
            pos.append(p0 + i)
            seq.append(s)
            kind.append(1 if n == 1 else 2)
            off.append(i)
            slot.append(int(perm[s, (p0 + i) // block_size]) * block_size + (p0 + i) % block_size)
    while len(pos) % 16:
        pos.append(0); seq.append(0); kind.append(0); off.append(0); slot.append(-1)  # noqa: E702
    blk, tile, one = blk or [(0, 0, 0, 0)], tile + [(0, 0, 0, 0)] * 3, one + [-1] * 2
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)  # noqa: E731
    st = mx.Step(i32(pos), i32(pos), i32(slot), i32(seq), i32(kind), i32(off), i32(perm.tolist()), i32(one), i32(seg).t().contiguous(), i32(blk).t().contiguous(), len(blk),
                   i32(tile).t().contiguous(), len(tile) - 1, all(n == 1 for n, _, _ in portions), long)
    st.chunks, st.n_chunks, st.first_chunk = i32(chunk + [(0, 0, 0, 0)] * 2).t().contiguous(), len(chunk) + 1, i32(first_chunk)
    if reach:
        at, spans, lb = 3, [[0] * smax for _ in range(3)], []
        for row, n, p0, s, _t in seg[::-1]:
            if n == 1:
                continue
            lo = max(0, p0 - reach + 1)
            spans[0][s], spans[1][s], spans[2][s] = at, lo, p0 + n - lo
            lb += [(row + o, min(128, n - o), p0 + o, at - lo) for o in range(0, n, 128)]
            at += p0 + n - lo
        lb += [(0, 0, 0, 0)] * 2
        st.spans, st.span_rows, st.latent_blocks, st.n_latent_blocks = i32(spans), at + 5, i32(lb).t().contiguous(), len(lb) - 1
    return st


def rel(got, want):
    return float((got.double().cpu() - want).norm() / want.norm())


def replay(path, backend, tokens_=1024, graphs=False):
    rp = Replay(engine_for(path, backend[1], tokens_, backend[0], graphs=graphs))
    if graphs:
        rp.engine.warmup()
    return rp
