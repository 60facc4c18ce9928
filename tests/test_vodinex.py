"""The Vodinex design through the engine against the plain model of tests/vodinex_oracle.py: every mechanism alone, prompts,
decoding, portions, batches, re-used pages and slots, greedy generation.  Each test runs on the CPU ops, and (marked gpu) on the
HIP kernels in fp32 and bf16."""

import json
import math
import os
import subprocess
import sys

import pytest
import torch
import vodinex_oracle as oracle
from hybrid_testing import BACKENDS, ROOT, TYPES, close, feed, make_step, mixers_of, rel, replay, save, tokens

from kvmini.engine.engine import EngineConfig, LLMEngine
from kvmini.engine.replay import engine_for
from kvmini.engine.scheduler import SamplingParams
from kvmini.models import hybrid, registry, vodinex

# ---- configurations: sizes, head ratios, layer orders and constants of their own
def attn(heads, kv, dim, vdim, chunk, rot, scale=None, base=10000.0):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "mask": {"size": chunk}, "rot": {"base": base, "dims": rot}, "scale": dim ** -0.5 if scale is None else scale}


def delta(heads, kv, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}


def par(left, right, ff, ls, rs):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": ls, "right_scale": rs}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def alone(d, ff):
    return {"type": "channel_delta", "mixer": d, "mlp": {"kind": "dense", "ff": ff} if ff else None}


CONFIGS = {
    # odd sizes, partly rotated heads, shared key heads in both branches, three taps
    "odd": dict(vocab=131, width=72, norm={"eps": 1e-5}, residual_mult=0.7,
                layers=[alone(delta(2, 1, 12, 20, 3), 0), par(attn(6, 2, 20, 12, 24, 8), delta(4, 2, 24, 16, 3), 100, 0.6, 1.3), par(attn(4, 4, 16, 28, 40, 16, base=700.0), delta(3, 3, 8, 12, 2), 0, 1.4, 0.5)]),
    # everything the odd model varies at its plain value; MLPs the other way round; a chunk of whole pages
    "plain": dict(vocab=200, width=64, norm={"eps": 1e-6}, residual_mult=1.0,
                  layers=[par(attn(2, 2, 32, 32, 32, 32), delta(2, 2, 32, 32, 4), 0, 1.0, 1.0), alone(delta(2, 2, 32, 32, 4), 96)]),
    # large heads, one key head, values wider than keys, columns that do not come in fours, one tap
    "wide": dict(vocab=97, width=140, norm={"eps": 1e-4}, residual_mult=0.4,
                 layers=[par(attn(3, 1, 96, 160, 20, 64, scale=0.2), delta(2, 1, 72, 6, 1), 40, 0.9, 1.2), par(attn(5, 1, 130, 70, 50, 0), delta(1, 1, 136, 36, 5), 64, 1.0, 2.0)]),
    # many query heads per key head, chunks shorter than a page, a parallel layer last without an MLP
    "many": dict(vocab=311, width=200, norm={"eps": 1e-5}, residual_mult=0.25,
                 layers=[par(attn(20, 1, 48, 80, 7, 24), delta(6, 3, 48, 40, 4), 264, 0.3, 0.8), alone(delta(5, 5, 80, 64, 4), 72), par(attn(9, 3, 64, 64, 30, 64, base=100.0), delta(2, 2, 16, 100, 2), 0, 1.0, 1.0)]),
    # one long chunk: contexts that decode steps share out over several workgroups
    "long": dict(vocab=83, width=48, norm={"eps": 1e-6}, residual_mult=0.8, layers=[par(attn(2, 1, 16, 24, 3000, 16), delta(1, 1, 16, 16, 2), 0, 1.0, 0.7)]),
}
RANKS = {"long": (4, 4), "many": (16, 24), "odd": (5, 7), "plain": (8, 8), "wide": (9, 3)}


def make_model(name, seed=0, sharp=0.0):
    """(config.json document, weights as float64 that are exact in bf16).  ``sharp`` scales the query / key norms, so that single
    keys dominate their softmax."""
    doc = dict(CONFIGS[name], architecture="Vodinex")
    cfg = vodinex.config_from_json(doc)
    shapes = hybrid.tensor_shapes(cfg)
    ra, rg = RANKS[name]
    gen = torch.Generator().manual_seed(seed)
    w = {}
    for n, s in shapes.items():
        s, leaf = list(s), n.rsplit(".", 1)[-1]
        if leaf in hybrid.RANKED:
            s[hybrid.RANKED[leaf]] = ra if leaf[0] == "a" else rg
        r = torch.randn(s, generator=gen, dtype=torch.float64)
        if "norm" in leaf:
            r = 1 + 0.2 * r
            if sharp and (n.endswith("q.norm") or n.endswith("k.norm")):
                r = r * sharp
        elif leaf == "conv":
            r = r / math.sqrt(s[1])
        elif leaf == "A_log":
            r = 0.5 * r - 0.5
        elif len(s) == 2 and n != "embed":
            r = r * 1.5 / math.sqrt(s[1])
        w[n] = r.to(torch.bfloat16).double()
    return doc, w


_built = {}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    def get(name, sharp=0.0):
        key = (name, sharp)
        if key not in _built:
            doc, w = make_model(name, seed=len(name), sharp=sharp)
            _built[key] = (save(tmp_path_factory.mktemp(name), doc, w), doc, w)
        return _built[key]

    return get


_want = {}


def want_logits(doc, w, toks, key):
    """The plain model's logits (a request is used by several tests)."""
    key = (key, tuple(toks))
    if key not in _want:
        _want[key] = oracle.logits(doc, w, toks)
    return _want[key]


# ---- mechanisms alone ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,kv,dim,vdim,chunk,rot", [(4, 2, 24, 20, 40, 16), (6, 2, 64, 40, 33, 48), (3, 1, 128, 64, 0, 32), (2, 2, 128, 128, 16, 128), (6, 3, 96, 128, 150, 0), (9, 1, 40, 256, 64, 40),
                                                         (2, 1, 300, 70, 48, 20), (20, 1, 64, 64, 7, 32), (12, 1, 128, 120, 5, 0), (36, 2, 80, 64, 100, 80)])
def test_chunked_attention_alone(backend, heads, kv, dim, vdim, chunk, rot):
    """One attention branch over a prompt in three portions, then single tokens.  Scores are sharp (large scale), and for some
    queries one key is made to stand out: far back, at page borders, and on both sides of chunk edges."""
    device, dtype = backend
    ty, mx = TYPES[dtype], mixers_of(device)
    t, eps = 190, 1e-5
    m = hybrid.AttentionSpec(heads, kv, dim, vdim, 6.0 / math.sqrt(dim), chunk, 10000.0, rot)
    gen = torch.Generator().manual_seed(dim + vdim)
    rnd = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()  # noqa: E731
    q, k, v, gl = rnd(t, heads * dim), rnd(t, kv * dim), rnd(t, kv * vdim), rnd(t, heads)
    c = chunk or t
    for i, j in [(i, j) for e in range(0, t, c) for i, j in ((e, e - 1), (e + 1, e), (e + c - 1, e), (e + 5, e - 3))] + [(17, 15), (31, 16), (160, 1), (189, 63)]:
        if 0 <= j <= i < t:
            for h in range(heads):  # (the rotation of the two differs; without one the score is the largest possible)
                q[i, h * dim : (h + 1) * dim] = k[j, (h // (heads // kv)) * dim : (h // (heads // kv) + 1) * dim]
    qn, kn, bias = 1 + 0.2 * rnd(dim), 1 + 0.2 * rnd(dim), 0.3 * rnd(heads * dim + kv * dim + kv * vdim)
    nq, nk = heads * dim, kv * dim
    want_q = oracle.rotate_half_pairs(oracle.rms_unit((q + bias[:nq]).view(t, heads, dim), eps) * qn, 10000.0, rot)
    want_k = oracle.rotate_half_pairs(oracle.rms_unit((k + bias[nq : nq + nk]).view(t, kv, dim), eps) * kn, 10000.0, rot)
    want = oracle.chunked_softmax_attention(want_q, want_k, (v + bias[nq + nk :]).view(t, kv, vdim), m.scale, chunk or 1 << 30) * torch.sigmoid(gl)[:, :, None] * 0.7
    pad8 = lambda x: torch.nn.functional.pad(x, (0, -x.shape[1] % 8))  # noqa: E731
    parts = [pad8(q), pad8(k), pad8(v), pad8(gl)]
    offs = [0, *torch.tensor([p.shape[1] for p in parts]).cumsum(0).tolist()]
    proj = torch.cat(parts, 1).to(ty).to(device)
    w = hybrid.AttentionWeights(offs[0], offs[1], offs[2], offs[3], 8, bias.float().to(device), qn.float().to(device), kn.float().to(device))
    pk, pv = mx.head_pads(dim, vdim, ty)
    cache = (torch.full((64, kv, 16, pk), 3.0, dtype=ty, device=device), torch.full((64, kv, 16, pv), -2.0, dtype=ty, device=device))
    half = rot // 2
    ang = torch.arange(256, dtype=torch.float64)[:, None] * 10000.0 ** (-2.0 * torch.arange(half, dtype=torch.float64) / max(1, rot))
    tabs = (ang.cos().float().to(device), ang.sin().float().to(device))
    got, at = torch.zeros(t, heads * vdim, dtype=torch.float64), 0
    for n in [70, 37, 2, 1, 73] + [1] * 7:
        st = make_step(mx, [(n, at, 2)], device, long=at % 2 == 1)
        x = torch.zeros(st.rows, proj.shape[1], dtype=ty, device=device)
        x[:n] = proj[at : at + n]
        mix = torch.zeros(st.rows, 8 + heads * vdim, dtype=ty, device=device)
        mx.attention(m, w, 0.7, eps, x, mix, cache, tabs, st)
        got[at : at + n] = mix[:n, 8:].double().cpu()
        at += n
    assert at == t and rel(got, want.reshape(t, -1)) < (2e-6 if dtype == "fp32" else 0.02)
    rows = (got - want.reshape(t, -1)).norm(dim=1) / want.reshape(t, -1).norm(dim=1)
    assert float(rows.max()) < (2e-5 if dtype == "fp32" else 0.08), int(rows.argmax())


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,kv,dim,vdim,taps,strong", [(4, 2, 24, 16, 3, 0.0), (2, 2, 128, 128, 4, 0.0), (3, 1, 40, 6, 1, 3.0), (4, 4, 28, 36, 2, 4.0), (2, 1, 200, 48, 6, 1.0), (8, 2, 64, 256, 4, 0.0), (2, 2, 256, 128, 3, 0.0), (1, 1, 260, 64, 4, 0.0)])
def test_delta_rule_alone(backend, heads, kv, dim, vdim, taps, strong):
    """One delta-rule branch: a prompt in portions (down to two tokens) beside another sequence's, then single tokens; decays from
    nearly one down to e^-60 per token (``strong``)."""
    device, dtype = backend
    ty, mx = TYPES[dtype], mixers_of(device)
    t, eps = 90, 1e-5
    m = hybrid.DeltaSpec(heads, kv, dim, vdim, taps)
    gen = torch.Generator().manual_seed(dim + vdim + taps)
    rnd = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()  # noqa: E731
    q, k, v, b = rnd(t, kv * dim), rnd(t, kv * dim), rnd(t, heads * vdim), 2 * rnd(t, heads)
    z, gl = 3 * rnd(t, heads * dim), rnd(t, heads * vdim)
    cq, ck, cv = rnd(kv * dim, taps), rnd(kv * dim, taps), rnd(heads * vdim, taps)
    a_log, dt, nw = rnd(heads) - 2 + strong, rnd(heads * dim) - 2, 1 + 0.2 * rnd(vdim)
    act = [oracle.short_conv_silu(x, c) for x, c in ((q, cq), (k, ck), (v, cv))]
    o = oracle.delta_recurrence(oracle.unit_vectors(act[0].view(t, kv, dim)) * dim ** -0.5, oracle.unit_vectors(act[1].view(t, kv, dim)), act[2].view(t, heads, vdim), torch.sigmoid(b),
                                oracle.channel_decay(z, a_log, dt, heads, dim))
    want = (oracle.rms_unit(o, eps) * nw * torch.sigmoid(gl).view(t, heads, vdim) * 1.3).reshape(t, -1)
    pad8 = lambda x: torch.nn.functional.pad(x, (0, -x.shape[1] % 8))  # noqa: E731
    parts, lows = [pad8(q), pad8(k), pad8(v), pad8(b)], [pad8(z), pad8(gl)]
    offs = [0, *torch.tensor([p.shape[1] for p in parts]).cumsum(0).tolist()]
    proj, low = torch.cat(parts, 1).to(ty).to(device), torch.cat(lows, 1).to(ty).to(device)
    f = lambda x: x.float().contiguous().to(device)  # noqa: E731
    w = hybrid.DeltaWeights(offs[0], offs[1], offs[2], offs[3], 0, 0, 0, lows[0].shape[1], 16, None, f(torch.cat((cq, ck, cv)).T), f(a_log), f(dt), f(nw))
    state = torch.full((4, heads, dim, vdim), 7.0, device=device)  # (left over from somebody else)
    ring = torch.full((4, taps, m.channels), 7.0, dtype=ty, device=device)
    ds = mx.DeltaState(m, w, 1.3, eps, state, ring)
    got, at = torch.zeros(2, t, heads * vdim, dtype=torch.float64), [0, 0]
    # (tokens of sequence A in slot 1, of sequence B in slot 3)
    for n in [(1, 0), (2, 5), (3, 1), (17, 16), (1, 33), (16, 2), (32, 2), (0, 3), (18, 28)]:
        ps = [(c, at[i], (1, 3)[i]) for i, c in enumerate(n) if c]
        st = make_step(mx, ps, device, n_blocks=80)
        rows = torch.cat([torch.arange(p0, p0 + c) for c, p0, _ in ps])
        x, lo = torch.zeros(st.rows, proj.shape[1], dtype=ty, device=device), torch.zeros(st.rows, low.shape[1], dtype=ty, device=device)
        x[: len(rows)], lo[: len(rows)] = proj[rows], low[rows]
        mix = torch.zeros(st.rows, 16 + heads * vdim, dtype=ty, device=device)
        ds.run(x, lo, mix, st)
        r = 0
        for i, c in enumerate(n):
            got[i, at[i] : at[i] + c] = mix[r : r + c, 16:].double().cpu()
            r += c
            at[i] += c
    assert at == [t, t]
    for i in range(2):
        rows = (got[i] - want).norm(dim=1) / want.norm(dim=1)
        assert rel(got[i], want) < (5e-6 if dtype == "fp32" else 0.01), i
        assert float(rows.max()) < (1e-4 if dtype == "fp32" else 0.05), (i, int(rows.argmax()))
    if device != "cpu":  # other slots are not touched
        assert bool((state[0] == 7).all()) and bool((state[2] == 7).all()) and bool((ring[0] == 7).all()) and bool((ring[2] == 7).all())


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width", [72, 300, 2048, 4500])
def test_gated_residual_and_embedding_alone(backend, width):
    device, dtype = backend
    ty, mx = TYPES[dtype], mixers_of(device)
    ld, t, eps, mult = hybrid.pad_k(width), 21, 1e-3, 0.45
    gen = torch.Generator().manual_seed(width)
    rnd = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()  # noqa: E731
    table, ids = rnd(50, width), torch.randint(0, 50, (t,), generator=gen)
    feed_, prev = torch.zeros(t, dtype=torch.int32), torch.tensor([9, 4, 49], dtype=torch.int64)
    feed_[3], feed_[7] = 2, 3  # from the previous step's ids
    x, xb, _keep = mx.embed_stream(table.to(ty).to(device), ids.int().to(device), feed_.to(device), prev.to(device), ld)
    ids[3], ids[7] = 4, 49
    assert torch.equal(x[:, :width].double().cpu(), table[ids]) and torch.equal(xb.float(), x) and bool((x[:, width:] == 0).all())
    y, b, gt, gb, g, fg = rnd(t, width), rnd(width), rnd(t, width), rnd(width), rnd(1), rnd(1)
    pad = lambda v: torch.nn.functional.pad(v, (0, ld - width))  # noqa: E731
    p32 = lambda v: pad(v).float().to(device)  # noqa: E731
    r = (y + b) * torch.sigmoid(gt + gb)
    want = table[ids] + mult * oracle.scalar_norm(r, g, eps)
    x0 = x.clone()
    out = mx.gated_residual(x, pad(y).to(ty).to(device), p32(b), pad(gt).to(ty).to(device), p32(gb), g.float().to(device), mult, eps, width, ty)
    assert rel(x[:, :width], want) < 1e-6 and rel(out[:, :width], want) < (1e-6 if dtype == "fp32" else 4e-3) and bool((x[:, width:] == 0).all()) and bool((out[:, width:] == 0).all())
    fin = mx.gated_residual(x0, pad(y).to(ty).to(device), p32(b), pad(gt).to(ty).to(device), p32(gb), g.float().to(device), mult, eps, width, ty, fg.float().to(device))
    assert rel(fin[:, :width], oracle.scalar_norm(want, fg, eps)) < (1e-6 if dtype == "fp32" else 4e-3)
    if device != "cpu":  # split-K partial sums instead of rows
        from kvmini.ops.hip_ops import Partial

        part = torch.randn(3, t, ld, generator=gen).to(device)
        part[2] = p32(y) - part[0] - part[1]
        gpart = torch.stack((p32(gt) * 0.25, p32(gt) * 0.75))
        x1 = table[ids].float().to(device)
        x1 = torch.nn.functional.pad(x1, (0, ld - width)).contiguous()
        mx.gated_residual(x1, Partial(part), p32(b), Partial(gpart), p32(gb), g.float().to(device), mult, eps, width, ty)
        assert rel(x1[:, :width], want) < 1e-5


@pytest.mark.parametrize("backend", BACKENDS)
def test_gelu_gated_projection_alone(backend):
    device, dtype = backend
    ty = TYPES[dtype]
    gen = torch.Generator().manual_seed(1)
    for rows in (16, 64, 96, 160):
        x = torch.randn(rows, 256, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()
        gate, up = ((torch.randn(136, 256, generator=gen, dtype=torch.float64) / 5).to(torch.bfloat16).double() for _ in range(2))
        want = oracle.gelu_tanh(x @ gate.T) * (x @ up.T)
        wgu = hybrid.interleave_gate_up(gate.to(ty), up.to(ty)).contiguous().to(device)
        if device == "cpu":
            from kvmini.ops import torch_ops as ops
        else:
            from kvmini.ops import hip_ops as ops
        got = ops.linear_geglu(x.to(ty).to(device), registry._pack_for(device, ty, "auto")(wgu))
        assert rel(got, want) < (1e-6 if dtype == "fp32" else 6e-3), rows


# ---- the whole model ----------------------------------------------------------------------------------------------
@pytest.mark.parametrize("backend", BACKENDS)
def test_residual_stream_after_every_layer(backend, models):
    path, doc, w = models("odd")
    toks = tokens(45, doc["vocab"], 3)
    rp = replay(path, backend)
    got = []
    rp.engine.runner._after_layer = lambda li, x: got.append(x[: len(toks), : doc["width"]].double().cpu())
    rp.step([{"id": 0, "tokens": toks, "want": [0]}], [0])
    want = oracle.layer_outputs(doc, w, toks)
    assert len(got) == len(want)
    for li, (a, b) in enumerate(zip(got, want)):
        assert rel(a, b) < (2e-6 if backend[1] == "fp32" else 0.02), li


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", [n for n in CONFIGS if n != "long"])
def test_prompts_portions_and_decoding_agree_with_the_plain_model(backend, name, models):
    """One request whole, in portions of changing size (down to two tokens, cut in the middle of pages and chunks), and token by
    token: the same logits everywhere."""
    path, doc, w = models(name, 2.0)
    toks = tokens(86, doc["vocab"], 7)
    want = want_logits(doc, w, toks, name)
    rp = replay(path, backend)
    for plan in ([86], [2, 3, 17, 2, 30, 5, 2, 25], [50] + [1] * 36, [1] * 86, [33, 1, 2, 1, 49]):
        got = feed(rp, [[(0, n)] for n in plan], {0: toks})[0]
        close(got, want, backend[1], (name, plan))


@pytest.mark.parametrize("backend", BACKENDS)
def test_batches_of_unequal_requests_and_reused_pages_and_slots(backend, models):
    """Up to four live requests, portions beside single tokens, in a pool that just holds them; pages and slots of finished requests
    go to new ones.  Each request's logits are those of the request alone."""
    path, doc, w = models("odd", 2.0)
    reqs = {i: tokens(n, doc["vocab"], 20 + i) for i, n in enumerate([61, 86, 1, 23, 64, 48, 2, 70])}
    plan = [[(0, 16), (1, 3), (2, 1)], [(0, 1), (3, 20)], [(1, 40), (0, 30), (3, 1)], [(0, 13), (3, 1), (1, 1)], [(0, 1), (3, 1), (1, 41)], [(1, 1), (4, 33)], [(4, 2), (5, 47), (6, 2)],
            [(4, 1), (5, 1), (7, 35)], [(4, 28), (7, 2)], [(7, 33)]]
    for seed in range(2):
        rp = replay(path, backend, 64 * 4, graphs=seed == 1)
        for _ in range(2):  # (the second time round every page and slot has been somebody else's)
            got = feed(rp, plan, reqs)
            for i, toks in reqs.items():
                close(got[i], want_logits(doc, w, toks, "odd"), backend[1], i)
        assert rp.engine.bm.num_free == rp.engine.bm.num_blocks - 1 and len(rp.engine.scheduler._free_slots) == 4 and not rp.live


@pytest.mark.parametrize("backend", BACKENDS)
def test_long_decoding(backend, models):
    """Decoding across many pages and several chunks, one token a step."""
    path, doc, w = models("plain", 2.0)
    toks = tokens(150, doc["vocab"], 9)
    got = feed(replay(path, backend, graphs=True), [[(0, 6)]] + [[(0, 1)]] * 144, {0: toks})[0]
    close(got, want_logits(doc, w, toks, "plain"), backend[1])


@pytest.mark.parametrize("backend", BACKENDS[:2])
def test_greedy_generation_through_the_scheduler(backend, models):
    """The engine's own entry point: prompts longer than a step's budget, more requests than slots, launch-ahead stepping, and a pool
    so small that sequences are preempted and start over — the plain model's greedy continuations."""
    device, dtype = backend
    path, doc, w = models("plain")
    prompts = [tokens(n, doc["vocab"], 40 + n) for n in (1, 5, 38, 60, 17)]
    n_new = 10
    want = [oracle.greedy(doc, w, p, n_new) for p in prompts]
    for blocks, ahead in ((0, True), (0, False), (7, True)):
        eng = LLMEngine(EngineConfig(model=path, device=device, dtype=dtype, max_num_seqs=3, max_batched_tokens=24, max_model_len=128, num_blocks=blocks, async_scheduling=ahead, launch_margin_ms=0.0))
        eng.warmup()
        assert eng.generate(prompts, SamplingParams(max_tokens=n_new)) == want, (blocks, ahead)
        assert eng.bm.prefix_hits == 0
        if blocks:
            assert eng.scheduler.num_preemptions > 0
        assert eng.generate(prompts[::-1], SamplingParams(max_tokens=n_new)) == want[::-1]
    out = eng.generate(prompts, SamplingParams(max_tokens=n_new, temperature=0.8, top_k=20, seed=5))
    assert out == eng.generate(prompts, SamplingParams(max_tokens=n_new, temperature=0.8, top_k=20, seed=5)) and all(0 <= t < doc["vocab"] for o in out for t in o)


@pytest.mark.gpu
def test_replayed_graphs_equal_eager_steps(models):
    """Every step shape of a mixed schedule, replayed several times with eager work in between, against the same steps without
    graphs: bit for bit."""
    path, doc, _w = models("odd")
    reqs = {i: tokens(n, doc["vocab"], 60 + i) for i, n in enumerate([70, 40, 90])}
    plan = [[(0, 20), (1, 10)], [(0, 1), (1, 1), (2, 50)], [(0, 1), (1, 1), (2, 1)], [(0, 1), (1, 1), (2, 2)], [(0, 47), (2, 1)], [(1, 27), (2, 36)]]
    a = replay(path, ("cuda:0", "bf16"), 256, graphs=True)
    b = replay(path, ("cuda:0", "bf16"), 256)
    assert a.engine.runner.graphs and not b.engine.runner.graphs
    for _ in range(3):
        ga, gb = feed(a, plan, reqs), feed(b, plan, reqs)
        assert all(torch.equal(ga[i], gb[i]) for i in reqs)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["bf16", "fp32"])
def test_long_contexts_in_one_chunk(models, dtype):
    """2100 tokens of context inside one chunk, beside a short request; decode steps (graphs) split the long context's keys."""
    path, doc, w = models("long", 3.0)
    reqs = {0: tokens(2112, doc["vocab"], 1), 1: tokens(40, doc["vocab"], 2)}
    rp = replay(path, ("cuda:0", dtype), 2304, graphs=True)
    kinds = []
    run = rp.engine.runner._run_staged
    rp.engine.runner._run_staged = lambda t_pad, max_ctx, kind=0, *a: (kinds.append(kind), run(t_pad, max_ctx, kind, *a))[1]
    got = feed(rp, [[(0, 1500), (1, 28)], [(0, 600)]] + [[(0, 1), (1, 1)]] * 12, reqs)
    assert kinds == [0, 0] + [2] * 12
    for i, toks in reqs.items():
        close(got[i], want_logits(doc, w, toks, "long"), dtype, i)


@pytest.mark.gpu
def test_generation_on_graphs_in_bf16_follows_the_plain_model(models):
    """bf16 serving (graphs, launch-ahead): each picked token is the plain model's best up to rounding."""
    path, doc, w = models("odd")
    eng = LLMEngine(EngineConfig(model=path, device="cuda:0", dtype="bf16", max_num_seqs=4, max_batched_tokens=64, max_model_len=128))
    eng.warmup()
    prompts = [tokens(n, doc["vocab"], 80 + n) for n in (3, 50, 9, 30, 77)]
    for p, o in zip(prompts, eng.generate(prompts, SamplingParams(max_tokens=12))):
        lg = oracle.logits(doc, w, p + o)[len(p) - 1 : -1]
        gap = lg.max(-1).values - lg.gather(1, torch.tensor(o)[:, None])[:, 0]
        assert len(o) == 12 and float(gap.max()) < 0.1 * float(lg.std()), gap
    hot = SamplingParams(max_tokens=12, temperature=0.9, top_k=30, top_p=0.95, seed=11)
    out = eng.generate(prompts, hot)
    assert out == eng.generate(prompts, hot) and all(len(o) == 12 and 0 <= min(o) and max(o) < doc["vocab"] for o in out)


# ---- the framework around it --------------------------------------------------------------------------------------
def test_registry_and_configuration(models):
    path, doc, _w = models("wide")
    cfg, wpath = registry.resolve_model(path)
    assert cfg.family == "vodinex" and wpath == path and cfg.recurrent and cfg.num_layers == 2
    left, right = cfg.layers[0].branches
    assert left.mixer == hybrid.AttentionSpec(3, 1, 96, 160, 0.2, 20, 10000.0, 64) and left.scale == 0.9 and right.scale == 1.2 and right.mixer.taps == 1
    assert registry.resolve_model("vodinex-tiny")[0].name == "vodinex-tiny" and registry.resolve_model("tiny")[0].name == "tiny" and "vodinex-8b" in registry.preset_names()
    bad = json.loads(json.dumps(doc))
    bad["layers"][0]["type"] = "something"
    with pytest.raises(ValueError, match="unknown mixer"):
        vodinex.config_from_json(bad)
    with pytest.raises(ValueError, match="architecture"):
        vodinex.config_from_json(dict(doc, architecture="Other"))


def test_checkpoints_that_do_not_fit_are_refused(models, tmp_path):
    _path, doc, w = models("plain")
    short = dict(w)
    del short["l1.mix.A_log"]
    with pytest.raises(KeyError, match="A_log"):
        engine_for(save(tmp_path / "a", doc, short), "fp32", 64, "cpu")
    with pytest.raises(ValueError, match="shape"):
        engine_for(save(tmp_path / "b", doc, dict(w, **{"l0.mix.left.k": w["l0.mix.left.k"][:-1]})), "fp32", 64, "cpu")


def test_what_a_recurrent_state_rules_out_is_refused():
    base = dict(model="vodinex-tiny", device="cpu", dtype="fp32", max_model_len=64, max_num_seqs=2)
    with pytest.raises(ValueError, match="recurrent"):
        LLMEngine(EngineConfig(**base, draft_model="tiny", num_speculative_tokens=2))
    with pytest.raises(ValueError, match="quantization"):
        LLMEngine(EngineConfig(**base, quantization="fp8"))
    with pytest.raises(ValueError, match="KV cache"):
        LLMEngine(EngineConfig(**base, kv_cache_dtype="fp8"))
    with pytest.raises(ValueError, match="tensor parallelism"):
        LLMEngine(EngineConfig(**base, tp_size=2))
    assert not LLMEngine(EngineConfig(**base)).bm.enable_prefix_caching


def test_replay_refuses_what_does_not_fit(models):
    path, doc, _w = models("plain")
    rp = replay(path, ("cpu", "fp32"), 64)
    with pytest.raises(ValueError, match="max_batched_tokens"):
        rp.step([{"id": 0, "tokens": tokens(65, doc["vocab"], 0), "want": []}], [])
    rp = replay(path, ("cpu", "fp32"), 128)
    for i in range(4):
        assert rp.step([{"id": i, "tokens": [1], "want": []}], []) is None
    with pytest.raises(ValueError, match="live requests"):
        rp.step([{"id": 9, "tokens": [1], "want": []}], [])
    with pytest.raises(ValueError, match="vocabulary"):
        rp.step([{"id": 0, "tokens": [doc["vocab"]], "want": []}], [])


def test_the_image_graphs_are_captured_on_lists_no_rows():
    """Warm-up and capture run on a staged image of padding rows: no row may be listed as a sequence's, it has no cache slot."""
    r = LLMEngine(EngineConfig(model="vodinex-tiny", device="cpu", dtype="fp32", max_model_len=64, max_num_seqs=3)).runner
    r._stage_dummy()
    assert bool((r._dev("singles") == -1).all()) and bool((r._dev("slots") == -1).all())
    for k in ("portions", "query_blocks", "tiles"):
        assert bool((r._dev(k).view(5 if k == "portions" else 4, -1)[1] == 0).all()), k
    assert torch.isfinite(r.forward(16)).all()


def test_trace_runner_program(models, tmp_path):
    """bin/trace_run as a user calls it (reference ops on the CPU)."""
    import numpy as np

    path, doc, w = models("odd", 2.0)
    toks = tokens(64, doc["vocab"], 20 + 4)
    lines = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:30], "want": [0, 29]}], "end": []}, {"step": 1, "entries": [{"id": "x", "tokens": toks[30:50], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": toks[50:51], "want": [0]}], "end": ["x"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64", "--device", "cpu"],
                       input="\n".join(json.dumps(x) for x in lines) + "\n", capture_output=True, text=True, timeout=120)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    assert not (tmp_path / "1.f32").exists()
    got = torch.from_numpy(np.concatenate([np.fromfile(tmp_path / f"{i}.f32", dtype="<f4").reshape(-1, doc["vocab"]) for i in (0, 2)]))
    close(got, want_logits(doc, w, toks, "odd")[[0, 29, 50]], "fp32")


def test_openai_server_on_a_hybrid_model():
    """The HTTP front-end: chat completion, guided JSON, seeded sampling with penalties and log-probabilities."""
    import urllib.request

    from kvmini.server.native import start_native_in_thread

    eng = LLMEngine(EngineConfig(model="vodinex-tiny", device="cpu", dtype="fp32", max_num_seqs=4, max_model_len=256, max_batched_tokens=64))
    _srv, url, stop = start_native_in_thread(eng, model_name="v")

    def post(**kw):
        body = json.dumps(dict({"model": "v", "messages": [{"role": "user", "content": "hi there"}]}, **kw)).encode()
        return json.loads(urllib.request.urlopen(urllib.request.Request(url + "/v1/chat/completions", body, {"Content-Type": "application/json"}), timeout=60).read())

    try:
        assert post(max_tokens=8)["usage"]["completion_tokens"] == 8
        assert isinstance(json.loads(post(max_tokens=40, response_format={"type": "json_object"})["choices"][0]["message"]["content"]), dict)
        kw = dict(max_tokens=8, temperature=0.7, seed=3, logprobs=True, top_logprobs=2, min_tokens=4, frequency_penalty=0.3)
        a, b = post(**kw)["choices"][0], post(**kw)["choices"][0]
        assert a["message"] == b["message"] and len(a["logprobs"]["content"]) == 8
    finally:
        stop()


def test_command_line_generation(models, tmp_path):
    path, doc, w = models("plain")
    out = tmp_path / "o.jsonl"
    r = subprocess.run([sys.executable, "-m", "kvmini", "generate", "--model", path, "--device", "cpu", "--dtype", "fp32", "--prompt", "hello there", "--max-tokens", "6", "--max-model-len", "128",
                        "--out", str(out)], capture_output=True, text=True, timeout=120, cwd=ROOT)
    assert r.returncode == 0, r.stderr[-2000:]
    from kvmini.engine.tokenizer import get_tokenizer

    prompt = get_tokenizer(doc["vocab"], 1, -1).encode("hello there", add_bos=True)
    assert json.loads(out.read_text().splitlines()[0])["token_ids"] == oracle.greedy(doc, w, prompt, 6)
