"""The Pipilix design through the engine against the plain model of tests/pipilix_oracle.py: every mechanism alone, prompts,
decoding, portions, batches, re-used pages and slots, loops, greedy generation.  Each test runs on the CPU ops, and (marked gpu)
on the HIP kernels in fp32 and bf16."""

import json
import math
import os
import subprocess
import sys

import pipilix_oracle as oracle
import pytest
import torch
from hybrid_testing import BACKENDS, ROOT, TYPES, close, feed, make_step, mixers_of, rel, replay, save, tokens

from kvmini.engine.engine import EngineConfig, LLMEngine
from kvmini.engine.replay import engine_for
from kvmini.engine.scheduler import SamplingParams
from kvmini.models import hybrid, pipilix, registry


# ---- configurations: sizes, layer orders, loops and constants of their own
def mix(heads, dim, vdim, rank, window, scale=None):
    return {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "mask": {"size": window}, "scale": dim ** -0.5 if scale is None else scale}


def layer(m, mlp=None):
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, limit):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit}}


CONFIGS = {
    # odd sizes everywhere, a loop in the middle, a layer without a feed-forward, mixtures of different sizes
    "odd": dict(vocab=131, width=75, norm={"eps": 1e-5}, embedding={"scale": 3.5}, logit_scale=0.7, loop={"start": 1, "stop": 3, "times": 3},
                layers=[layer(mix(3, 20, 12, 28, 24), moe(5, 2, 36, 0.8)), layer(mix(5, 12, 28, 44, 40), dense(100)), layer(mix(2, 36, 20, 12, 9), moe(7, 3, 20, 1.2)), layer(mix(4, 16, 16, 40, 33))]),
    # constants at their plain values: one pass of the loop, one head, one expert a token, windows of whole pages
    "plain": dict(vocab=200, width=64, norm={"eps": 1e-6}, embedding={"scale": 1.0}, logit_scale=1.0, loop={"start": 0, "stop": 2, "times": 1},
                  layers=[layer(mix(1, 32, 32, 64, 32), moe(4, 1, 32, 7.0)), layer(mix(2, 64, 64, 128, 16), dense(96))]),
    # large heads and latents (beyond one tile of the kernels), many experts chosen, a loop that ends the model, a window of one token
    "wide": dict(vocab=97, width=140, norm={"eps": 1e-4}, embedding={"scale": 0.5}, logit_scale=2.5, loop={"start": 2, "stop": 3, "times": 2},
                 layers=[layer(mix(2, 130, 70, 200, 50, 0.06), moe(20, 6, 44, 2.0)), layer(mix(3, 96, 160, 300, 1), dense(40)), layer(mix(20, 24, 8, 130, 70, 0.15), moe(3, 3, 60, 0.5))]),
    # no loop, sizes past the matrix-core kernels (heads above 256, latents above 512)
    "huge": dict(vocab=83, width=48, norm={"eps": 1e-5}, embedding={"scale": 2.0}, logit_scale=0.4, layers=[layer(mix(2, 300, 20, 96, 20, 0.06), dense(40)), layer(mix(1, 24, 40, 600, 30), moe(70, 4, 24, 1.0))]),
    # a window beyond two thousand tokens: contexts that decode steps share out over many workgroups
    "long": dict(vocab=83, width=48, norm={"eps": 1e-6}, embedding={"scale": 1.5}, logit_scale=1.0, loop={"start": 0, "stop": 1, "times": 2}, layers=[layer(mix(2, 16, 24, 40, 2050), dense(40))]),
}


def make_model(name, seed=0, sharp=1.0):
    """(config.json document, weights as float64 that are exact in bf16).  ``sharp`` scales the queries, so that single keys dominate
    their softmax."""
    doc = dict(CONFIGS[name], architecture="Pipilix")
    gen = torch.Generator().manual_seed(seed)
    w = {}
    for n, s in hybrid.tensor_shapes(pipilix.config_from_json(doc)).items():
        r = torch.randn(s, generator=gen, dtype=torch.float64)
        leaf = n.rsplit(".", 1)[-1]
        if leaf.startswith("norm"):
            r = 1 + 0.2 * r
        elif leaf == "correction":
            r = 0.3 * r
        elif leaf == "step":
            r = 0.5 * r
        elif n != "embed":
            r = r * 1.5 / math.sqrt(s[1]) * (sharp if n.endswith("mix.q") else 1.0)
        w[n] = r.to(torch.bfloat16).double()
    return doc, w


_built = {}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    def get(name, sharp=1.0):
        key = (name, sharp)
        if key not in _built:
            doc, w = make_model(name, seed=len(name), sharp=sharp)
            _built[key] = (save(tmp_path_factory.mktemp(name), doc, w), doc, w)
        return _built[key]

    return get


_requests = {}


def clear_choices(doc, w, n, seed, key, margin=0.008):
    """(request of n tokens, the plain model's logits): random tokens, changed where a choice of experts is so close that rounding could
    turn it (what follows would be another computation)."""
    key = (key, n, seed)
    if key not in _requests:
        toks = tokens(n, doc["vocab"], seed)
        for i in range(60 * n):
            tight = (oracle.closest_choices(doc, w, toks) < margin).nonzero().view(-1)
            if len(tight) == 0:
                break
            toks[int(tight[0])] = (toks[int(tight[0])] + 1 + i) % doc["vocab"]
        assert len(tight) == 0
        _requests[key] = (toks, oracle.logits(doc, w, toks))
    return _requests[key]


# ---- mechanisms alone ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width", [75, 300, 2048])
def test_embedding_with_sine_positions_alone(backend, width):
    device, dtype = backend
    ty, mx = TYPES[dtype], mixers_of(device)
    ld, t = hybrid.pad_k(width), 21
    gen = torch.Generator().manual_seed(width)
    table, ids = torch.randn(50, width, generator=gen, dtype=torch.float64).to(torch.bfloat16).double(), torch.randint(0, 50, (t,), generator=gen)
    feed_, prev = torch.zeros(t, dtype=torch.int32), torch.tensor([9, 4, 49], dtype=torch.int64)
    feed_[3] = 2
    first = [0, 1, 2, 3, 8191, 65537, 999983]  # (far positions: whole turns come off before rounding)
    pos = torch.tensor([first[i % 7] + i // 7 for i in range(t)], dtype=torch.int32)
    x, xb, keep = mx.embed_stream(table.to(ty).to(device), ids.int().to(device), feed_.to(device), prev.to(device), ld, 2.75, pos.to(device), True)
    ids[3] = 4
    want = table[ids] * 2.75 + torch.cat([oracle.sine_positions(1, width, int(p)) for p in pos])
    assert float((x[:, :width].double().cpu() - want).abs().max()) < 2e-6 and bool((x[:, width:] == 0).all())
    assert torch.equal(keep, x) and keep.data_ptr() != x.data_ptr() and torch.equal(xb, x.to(ty))


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width", [75, 300, 2048, 4500])
def test_residual_update_with_norms_on_both_sides_and_joining_rows(backend, width):
    device, dtype = backend
    ty, mx = TYPES[dtype], mixers_of(device)
    ld, t, eps, top = hybrid.pad_k(width), 19, 1e-3, 3
    gen = torch.Generator().manual_seed(width)
    rnd = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()  # noqa: E731
    x0, y, g, ng, jr, jv = rnd(t, width), rnd(t, width), 1 + 0.2 * rnd(width), 1 + 0.2 * rnd(width), rnd(t, width), rnd(width)
    p32 = lambda v: torch.nn.functional.pad(v, (0, ld - width)).float().contiguous().to(device)  # noqa: E731
    tol = 2e-6 if dtype == "fp32" else 4e-3
    new = x0 + oracle.rms_unit(y, eps) * g
    for join, joined in ((None, new), ((None, p32(jv)), new + jv), ((p32(jr), p32(jv)), new + jr + jv)):
        x = p32(x0)
        out = mx.gated_residual(x, p32(y).to(ty), None, None, None, p32(g), 1.0, eps, width, ty, p32(ng), join)
        assert rel(x[:, :width], joined) < 2e-6 and rel(out[:, :width], oracle.rms_unit(joined, eps) * ng) < tol
        assert bool((x[:, width:] == 0).all()) and bool((out[:, width:] == 0).all())
        x = p32(new)  # the second half alone
        assert rel(mx.stream_norm(x, join, p32(ng), eps, width, ty)[:, :width], oracle.rms_unit(joined, eps) * ng) < tol and rel(x[:, :width], joined) < 2e-6
    if device != "cpu":  # experts' rows instead: weight zero means that the row was never written
        rows, wt = rnd(t * top, width), torch.rand(t, top, generator=gen)
        wt[2, 1], wt[5] = 0, 0
        want = x0 + oracle.rms_unit((rows.view(t, top, width) * wt.double()[:, :, None]).sum(1), eps) * g
        dev = p32(rows).to(ty)
        dev[wt.view(-1).to(device) == 0] = float("nan")
        x = p32(x0)
        mx.gated_residual(x, mx.ExpertRows(dev, wt.to(device)), None, None, None, p32(g), 1.0, eps, width, ty, p32(ng))
        assert rel(x[:, :width], want) < 2e-6


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,dim,vdim,rank,window", [(4, 24, 20, 40, 37), (3, 64, 64, 128, 16), (2, 128, 128, 512, 64), (5, 100, 130, 300, 50), (17, 16, 8, 200, 1), (33, 40, 72, 130, 33),
                                                        (1, 200, 256, 512, 300), (2, 256, 40, 64, 2), (2, 300, 20, 96, 48), (1, 24, 40, 600, 31), (6, 48, 100, 256, 129)])
def test_latent_attention_alone(backend, heads, dim, vdim, rank, window):
    """One latent branch over a prompt in portions beside another sequence's, then single tokens.  For some queries one key is made to
    stand out: far back, at page borders, the first tokens, and just inside and just outside the window."""
    device, dtype = backend
    ty, mx = TYPES[dtype], mixers_of(device)
    t, eps = 330, 1e-5
    m = hybrid.LatentSpec(heads, dim, vdim, rank, 4.0 / math.sqrt(dim * rank), window)
    gen = torch.Generator().manual_seed(dim + vdim + rank)
    rnd = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()  # noqa: E731
    c, gl, cn = rnd(t, rank), rnd(t, heads), 1 + 0.2 * rnd(rank)
    uk, uv = rnd(heads * dim, rank), (rnd(heads * vdim, rank) / math.sqrt(rank)).to(torch.bfloat16).double()
    lat = oracle.rms_unit(c, eps) * cn
    k = (lat @ uk.T).view(t, heads, dim)
    q = rnd(t, heads * dim)
    for i in list(range(0, 60, 7)) + [95, 111, 127, 128, 129, 150, 200, 255, 256, 300, 323, 325, 327, 329]:
        for j in (i - window, i - window + 1, i - window + 2, 0, 1, (i // 16) * 16, (i // 16) * 16 - 1, i):
            if 0 <= j <= i and (i + j) % 3 == 0:
                a = k[j].reshape(-1)
                q[i] = (a / a.pow(2).mean().sqrt()).to(torch.bfloat16).double()
    want = oracle.windowed_softmax_attention(q.view(t, heads, dim), k, (lat @ uv.T).view(t, heads, vdim), m.scale, window) * torch.sigmoid(gl)[:, :, None] * 0.7
    want = want.reshape(t, -1)
    lay = registry._pack_for(device, ty, "auto")
    dkp, dvp, rkp = lay.latent_pads(m)
    pad = lambda x, n: torch.nn.functional.pad(x, (0, n - x.shape[-1]))  # noqa: E731
    parts = [pad(q.view(t, heads, dim), dkp).reshape(t, -1), pad(c, rkp), gl]
    parts = [pad(p, -(-p.shape[1] // 8) * 8) for p in parts]
    offs = [0, *torch.tensor([p.shape[1] for p in parts]).cumsum(0).tolist()]
    proj = torch.cat(parts, 1).to(ty).to(device)
    ukp = torch.nn.functional.pad(uk.view(heads, dim, rank), (0, rkp - rank, 0, dkp - dim)).to(ty).to(device)
    uvp = torch.nn.functional.pad(uv.view(heads, vdim, rank), (0, rkp - rank, 0, dvp - vdim)).to(ty).to(device)
    w = hybrid.LatentWeights(offs[0], offs[1], offs[2], 8, dkp, dvp, rkp, pad(cn, rkp).float().to(device), lay.heads(ukp.transpose(1, 2).contiguous(), m), lay.heads(uvp, m),
                             lay(torch.cat((ukp.reshape(-1, rkp), uvp.reshape(-1, rkp)))) if lay.expands(m) else None)
    cache = torch.full((128, 1, 16, rkp), 3.0, dtype=ty, device=device)  # (left over from somebody else)
    got, at = torch.zeros(2, t, heads * vdim, dtype=torch.float64), [0, 0]
    for n in [(70, 1), (37, 30), (2, 1), (1, 129), (150, 2), (3, 1), (2, 100), (55, 0), (0, 57)] + [(1, 1)] * 9 + [(1, 0)]:
        ps = [(x, at[i], (1, 3)[i]) for i, x in enumerate(n) if x]
        st = make_step(mx, ps, device, n_blocks=128, long=at[0] % 2 == 1, reach=window, per=24)
        rows = torch.cat([torch.arange(p0, p0 + x) for x, p0, _ in ps])
        x = torch.zeros(st.rows, proj.shape[1], dtype=ty, device=device)
        x[: len(rows)] = proj[rows.to(device)]
        out = torch.zeros(st.rows, 8 + heads * vdim, dtype=ty, device=device)
        mx.latent_attention(m, w, 0.7, eps, x, out, cache, st)
        r = 0
        for i, z in enumerate(n):
            got[i, at[i] : at[i] + z] = out[r : r + z, 8:].double().cpu()
            r += z
            at[i] += z
    assert at == [t, t]
    for i in range(2):
        rows = (got[i] - want).norm(dim=1) / want.norm(dim=1)
        assert rel(got[i], want) < (3e-6 if dtype == "fp32" else 0.02), i
        assert float(rows.max()) < (4e-5 if dtype == "fp32" else 0.08), (i, int(rows.argmax()))


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("experts,top,width,ff,limit,t", [(5, 2, 75, 36, 0.7, 20), (16, 1, 128, 64, 7.0, 1), (70, 6, 300, 100, 1.0, 77), (3, 3, 256, 40, 0.5, 128), (40, 4, 140, 72, 1.0, 200),
                                                          (8, 4, 256, 96, 2.0, 333), (2, 1, 140, 100, 1.0, 300), (300, 8, 64, 24, 1.0, 150), (1, 1, 64, 200, 1.0, 140)])
def test_experts_alone(backend, experts, top, width, ff, limit, t):
    """Mixtures in which the correction changes the choice and the clamps are hit; padding rows in between choose nobody."""
    device, dtype = backend
    ty, mx = TYPES[dtype], mixers_of(device)
    gen = torch.Generator().manual_seed(experts + ff)
    rnd = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()  # noqa: E731
    names = {"router": (experts, width), "correction": (experts,)}
    for e in range(experts):
        names.update({f"e{e}.gate": (ff, width), f"e{e}.up": (ff, width), f"e{e}.down": (width, ff)})
    w = {"m." + k: (rnd(*s) / math.sqrt(s[1]) if len(s) == 2 else 0.4 * rnd(*s)).to(torch.bfloat16).double() for k, s in names.items()}
    h = rnd(4 * t + 64, width)  # (rows with a clear choice, see below)
    z = h @ w["m.router"].T
    h = h[(oracle.choice_margin(z, w["m.correction"], top) > 1e-4).nonzero().view(-1)][:t]
    assert len(h) == t
    idx, _wt = oracle.choose_experts(h @ w["m.router"].T, w["m.correction"], top)
    if top < experts and experts > 2 and t > 1:
        assert not torch.equal(idx.sort(-1).values, torch.topk(h @ w["m.router"].T, top, -1).indices.sort(-1).values)
    want = oracle.mixture(h, w, "m", {"router": {"top": top}, "expert": {"limit": limit}})
    # through the weight packing of a whole layer
    cfg = hybrid.HybridConfig("m", 8, width, (hybrid.LayerSpec((hybrid.BranchSpec(hybrid.LatentSpec(1, 8, 8, 8, 1.0, 4), "mix"),), moe=hybrid.MoeSpec(experts, top, ff, limit)),), 1e-5, wiring="sandwich")
    shapes = hybrid.tensor_shapes(cfg)
    get = lambda n: w["m." + n[len("l0.mlp.") :]] if n.startswith("l0.mlp.") else torch.zeros(shapes[n])  # noqa: E731
    mw = hybrid.build_weights(cfg, get, ty, device, registry._pack_for(device, ty, "auto")).layers[0].moe
    rows = -(-(t + t // 5) // 16) * 16
    live = torch.tensor([i for i in range(rows) if i % 6 != 3][:t])
    st = make_step(mx, [(rows, 0, 0)], device, n_blocks=64, per=32)
    st.slots = torch.full((rows,), -1, dtype=torch.int32)
    st.slots[live] = 5
    st.slots = st.slots.to(device)
    x = torch.full((rows, cfg.ld), 2.0)
    x[live] = torch.nn.functional.pad(h, (0, cfg.ld - width)).float()
    y = mx.experts(cfg.layers[0].moe, mw, x.to(ty).to(device), st)
    if device != "cpu":
        dead = torch.ones(rows, dtype=torch.bool)
        dead[live] = False
        assert bool((y.weights[dead.to(device)] == 0).all())
        clean = torch.where(y.weights.view(-1, 1) == 0, torch.zeros_like(y.rows.float()), y.rows.float())
        y = (clean.view(rows, top, -1) * y.weights[:, :, None]).sum(1)
    assert rel(y[live.to(device), :width], want) < (3e-6 if dtype == "fp32" else 0.012)
    assert bool((y[live.to(device), width:] == 0).all())


@pytest.mark.parametrize("backend", BACKENDS)
def test_silu_gated_projection_alone(backend):
    device, dtype = backend
    ty = TYPES[dtype]
    gen = torch.Generator().manual_seed(1)
    if device == "cpu":
        from kvmini.ops import torch_ops as ops
    else:
        from kvmini.ops import hip_ops as ops
    for rows in (16, 96, 160):
        x = torch.randn(rows, 256, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()
        gate, up = ((torch.randn(136, 256, generator=gen, dtype=torch.float64) / 5).to(torch.bfloat16).double() for _ in range(2))
        wgu = hybrid.interleave_gate_up(gate.to(ty), up.to(ty)).contiguous().to(device)
        z = x @ gate.T
        got = ops.linear_swiglu(x.to(ty).to(device), registry._pack_for(device, ty, "auto")(wgu))
        assert rel(got, z * torch.sigmoid(z) * (x @ up.T)) < (1e-6 if dtype == "fp32" else 6e-3), rows


# ---- the whole model ----------------------------------------------------------------------------------------------
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["odd", "wide", "huge"])
def test_residual_stream_after_every_layer_run(backend, name, models):
    path, doc, w = models(name)
    toks, _ = clear_choices(doc, w, 45, 3, name)
    rp = replay(path, backend)
    got = []
    rp.engine.runner._after_layer = lambda ri, x: got.append(x[: len(toks), : doc["width"]].double().cpu().clone())
    rp.step([{"id": 0, "tokens": toks, "want": [0]}], [0])
    want = oracle.layer_outputs(doc, w, toks)
    assert len(got) == len(want) == len(rp.engine.mcfg.runs)
    for ri, (a, b) in enumerate(zip(got, want)):
        assert rel(a, b) < (3e-6 if backend[1] == "fp32" else 0.02), ri


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", [n for n in CONFIGS if n != "long"])
def test_prompts_portions_and_decoding_agree_with_the_plain_model(backend, name, models):
    """One request whole, in portions of changing size (down to two tokens, cut in the middle of pages and windows), and token by
    token: the same logits everywhere."""
    path, doc, w = models(name, 2.0)
    toks, want = clear_choices(doc, w, 86, 7, name)
    rp = replay(path, backend)
    for plan in ([86], [2, 3, 17, 2, 30, 5, 2, 25], [50] + [1] * 36, [1] * 86, [33, 1, 2, 1, 49]):
        got = feed(rp, [[(0, n)] for n in plan], {0: toks})[0]
        close(got, want, backend[1], (name, plan))


@pytest.mark.parametrize("backend", BACKENDS)
def test_batches_of_unequal_requests_and_reused_pages_and_slots(backend, models):
    """Up to four live requests, portions beside single tokens, in a pool that just holds them; pages and slots of finished requests
    go to new ones.  Each request's logits are those of the request alone."""
    path, doc, w = models("odd", 2.0)
    sizes = [61, 86, 1, 23, 64, 48, 2, 70]
    reqs = {i: clear_choices(doc, w, n, 20 + i, "odd") for i, n in enumerate(sizes)}
    plan = [[(0, 16), (1, 3), (2, 1)], [(0, 1), (3, 20)], [(1, 40), (0, 30), (3, 1)], [(0, 13), (3, 1), (1, 1)], [(0, 1), (3, 1), (1, 41)], [(1, 1), (4, 33)], [(4, 2), (5, 47), (6, 2)],
            [(4, 1), (5, 1), (7, 35)], [(4, 28), (7, 2)], [(7, 33)]]
    for seed in range(2):
        rp = replay(path, backend, 64 * 4, graphs=seed == 1)
        for _ in range(2):  # (the second time round every page and slot has been somebody else's)
            got = feed(rp, plan, {i: r[0] for i, r in reqs.items()})
            for i, (_toks, want) in reqs.items():
                close(got[i], want, backend[1], i)
        assert rp.engine.bm.num_free == rp.engine.bm.num_blocks - 1 and len(rp.engine.scheduler._free_slots) == 4 and not rp.live


@pytest.mark.parametrize("backend", BACKENDS)
def test_long_decoding(backend, models):
    """Decoding across many pages and several windows, one token a step."""
    path, doc, w = models("plain", 2.0)
    toks, want = clear_choices(doc, w, 150, 9, "plain")
    got = feed(replay(path, backend, graphs=True), [[(0, 6)]] + [[(0, 1)]] * 144, {0: toks})[0]
    close(got, want, backend[1])


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
        if blocks:
            assert eng.scheduler.num_preemptions > 0
        assert eng.generate(prompts[::-1], SamplingParams(max_tokens=n_new)) == want[::-1]
        if not blocks:
            assert eng.bm.prefix_hits > 0  # (latents are all there is to a prefix: the second round takes its blocks over)
    out = eng.generate(prompts, SamplingParams(max_tokens=n_new, temperature=0.8, top_k=20, seed=5))
    assert out == eng.generate(prompts, SamplingParams(max_tokens=n_new, temperature=0.8, top_k=20, seed=5)) and all(0 <= t < doc["vocab"] for o in out for t in o)


@pytest.mark.parametrize("backend", BACKENDS[:2])
def test_prefixes_are_shared_and_drafts_verified(backend):
    """What paged latents allow: requests with a common start, and steps that verify a draft model's tokens; greedy results stay."""
    device, dtype = backend
    base = dict(model="pipilix-tiny", device=device, dtype=dtype, max_num_seqs=4, max_batched_tokens=64, max_model_len=160)
    head = tokens(50, 512, 1)
    prompts = [head + tokens(n, 512, n) for n in (3, 20, 9)] + [head[:33]]
    plain = LLMEngine(EngineConfig(**base, enable_prefix_caching=False)).generate(prompts, SamplingParams(max_tokens=12, ignore_eos=True))
    eng = LLMEngine(EngineConfig(**base))
    assert [eng.generate([p], SamplingParams(max_tokens=12, ignore_eos=True))[0] for p in prompts] == plain and eng.bm.prefix_hits >= 3
    if device != "cpu":
        return  # (a draft of the other family runs in bf16 there, whose greedy results are not the fp32 model's)
    spec = LLMEngine(EngineConfig(**base, draft_model="tiny-draft", num_speculative_tokens=3))
    assert spec.generate(prompts, SamplingParams(max_tokens=12, ignore_eos=True)) == plain and spec.stats.spec_proposed > 0
    with pytest.raises(ValueError, match="self-speculation"):
        LLMEngine(EngineConfig(**base, draft_model="self:1", num_speculative_tokens=2))


@pytest.mark.gpu
def test_replayed_graphs_equal_eager_steps(models):
    """Every step shape of a mixed schedule — also portions deep inside their request, whose workspace is larger than the step's —
    replayed several times with eager work in between, against the same steps without graphs: bit for bit."""
    path, doc, _w = models("odd")
    reqs = {i: tokens(n, doc["vocab"], 60 + i) for i, n in enumerate([70, 40, 90])}
    plan = [[(0, 20), (1, 10)], [(0, 1), (1, 1), (2, 50)], [(0, 1), (1, 1), (2, 1)], [(0, 1), (1, 1), (2, 2)], [(0, 47), (2, 1)], [(1, 2), (2, 2)], [(1, 25), (2, 34)]]
    a = replay(path, ("cuda:0", "bf16"), 256, graphs=True)
    b = replay(path, ("cuda:0", "bf16"), 256)
    assert a.engine.runner.graphs and not b.engine.runner.graphs
    for _ in range(4):
        ga, gb = feed(a, plan, reqs), feed(b, plan, reqs)
        assert all(torch.equal(ga[i], gb[i]) for i in reqs)
    assert a.engine.runner.variant_graph_steps > 0


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["bf16", "fp32"])
def test_long_contexts_in_one_window(models, dtype):
    """More than 2050 tokens of context in one window, beside a short request, in prompts and in decode steps (graphs) that share the
    context's keys out."""
    path, doc, w = models("long", 3.0)
    reqs = {0: tokens(2112, doc["vocab"], 1), 1: tokens(40, doc["vocab"], 2)}
    rp = replay(path, ("cuda:0", dtype), 2304, graphs=True)
    kinds = []
    run = rp.engine.runner._run_staged
    rp.engine.runner._run_staged = lambda t_pad, max_ctx, kind=0, *a: (kinds.append(kind), run(t_pad, max_ctx, kind, *a))[1]
    got = feed(rp, [[(0, 1500), (1, 28)], [(0, 600)]] + [[(0, 1), (1, 1)]] * 12, reqs)
    assert kinds == [0, 0] + [2] * 12
    for i, toks in reqs.items():
        close(got[i], oracle.logits(doc, w, toks), dtype, i)


@pytest.mark.gpu
def test_generation_on_graphs_in_bf16_follows_the_plain_model(models):
    """bf16 serving (graphs, launch-ahead): each picked token is the plain model's best up to rounding."""
    path, doc, w = models("plain")
    eng = LLMEngine(EngineConfig(model=path, device="cuda:0", dtype="bf16", max_num_seqs=4, max_batched_tokens=64, max_model_len=128))
    eng.warmup()
    prompts = [clear_choices(doc, w, n, 80 + n, "plain")[0] for n in (3, 50, 9, 30, 77)]
    for p, o in zip(prompts, eng.generate(prompts, SamplingParams(max_tokens=12))):
        lg = oracle.logits(doc, w, p + o)[len(p) - 1 : -1]
        gap = lg.max(-1).values - lg.gather(1, torch.tensor(o)[:, None])[:, 0]
        n = int((oracle.closest_choices(doc, w, p + o)[len(p) :] < 0.008).long().cumsum(0).eq(0).sum())  # (up to a choice that rounding can turn)
        assert len(o) == 12 and float(gap[: n + 1].max()) < 0.1 * float(lg.std()), gap
    hot = SamplingParams(max_tokens=12, temperature=0.9, top_k=30, top_p=0.95, seed=11)
    out = eng.generate(prompts, hot)
    assert out == eng.generate(prompts, hot) and all(len(o) == 12 and 0 <= min(o) and max(o) < doc["vocab"] for o in out)


# ---- the framework around it --------------------------------------------------------------------------------------
def test_registry_and_configuration(models):
    path, doc, _w = models("odd")
    cfg, wpath = registry.resolve_model(path)
    assert cfg.family == "pipilix" and wpath == path and not cfg.recurrent and cfg.num_layers == 4
    assert cfg.layers[0].branches[0].mixer == hybrid.LatentSpec(3, 20, 12, 28, 20 ** -0.5, 24) and cfg.layers[0].moe == hybrid.MoeSpec(5, 2, 36, 0.8) and cfg.layers[3].moe is None
    assert [(r.layer, r.begins) for r in cfg.runs] == [(0, -1), (1, 0), (2, -1), (1, 1), (2, -1), (1, 2), (2, -1), (3, -1)]
    assert [(r.layer, None if r.begins < 0 else r.begins) for r in cfg.runs] == oracle.layer_order(doc)
    assert registry.resolve_model("pipilix-tiny")[0].name == "pipilix-tiny" and {"pipilix-1b", "pipilix-8b", "vodinex-8b"} <= set(registry.preset_names())
    for key, val, why in (("type", "something", "unknown mixer"), ("mlp", {"kind": "sparse"}, "unknown feed-forward")):
        bad = json.loads(json.dumps(doc))
        bad["layers"][0][key] = val
        with pytest.raises(ValueError, match=why):
            pipilix.config_from_json(bad)
    with pytest.raises(ValueError, match="architecture"):
        pipilix.config_from_json(dict(doc, architecture="Other"))
    with pytest.raises(ValueError, match="loop"):
        hybrid.check_config(pipilix.config_from_json(dict(doc, loop={"start": 3, "stop": 9, "times": 2})))
    with pytest.raises(ValueError, match="experts"):
        hybrid.check_config(pipilix.config_from_json(dict(doc, layers=[layer(mix(1, 8, 8, 8, 4), moe(3, 4, 8, 1.0))], loop=None)))


def test_checkpoints_that_do_not_fit_are_refused(models, tmp_path):
    _path, doc, w = models("plain")
    short = dict(w)
    del short["l0.mlp.e2.up"]
    with pytest.raises(KeyError, match="e2.up"):
        engine_for(save(tmp_path / "a", doc, short), "fp32", 64, "cpu")
    with pytest.raises(ValueError, match="shape"):
        engine_for(save(tmp_path / "b", doc, dict(w, **{"l0.mix.uk": w["l0.mix.uk"][:-1]})), "fp32", 64, "cpu")


def test_what_is_not_available_is_refused_by_name():
    base = dict(model="pipilix-tiny", device="cpu", dtype="fp32", max_model_len=64, max_num_seqs=2)
    for more, why in ((dict(quantization="fp8"), "quantization"), (dict(kv_cache_dtype="fp8"), "KV cache"), (dict(tp_size=2), "tensor parallelism")):
        with pytest.raises(ValueError, match=why):
            LLMEngine(EngineConfig(**base, **more))


def test_workspace_of_prompt_portions_is_staged_for_what_their_windows_reach():
    """Rows, positions and query blocks of the expansion workspace, and the step variant they ask for."""
    r = LLMEngine(EngineConfig(model="pipilix-tiny", device="cpu", dtype="fp32", max_model_len=512, max_num_seqs=4, max_batched_tokens=256)).runner
    r.expands = True  # (as on a GPU in bf16)
    r.max_latent_blocks = 256 // 128 + 4
    r._off["spans"], r._off["latent_blocks"] = (0, 12), (12, 4 * r.max_latent_blocks)
    st = torch.full((12 + 4 * r.max_latent_blocks,), -7, dtype=torch.int32).numpy()
    r._stage_spans(st, [(0, 1, 40, 2), (1, 130, 100, 1), (131, 5, 0, 3), (136, 2, 7, 0)])
    spans, blocks = st[:12].reshape(3, 4), st[12:].reshape(4, -1)
    assert r.reach == 20
    assert spans[:, 2].tolist() == [0, 0, 0] and spans[:, 1].tolist() == [0, 81, 149] and spans[:, 3].tolist() == [149, 0, 5] and spans[:, 0].tolist() == [154, 0, 9]
    assert blocks[:, :4].T.tolist() == [[1, 128, 100, -81], [129, 2, 228, -81], [131, 5, 0, 149], [136, 2, 7, 154]] and (blocks[1, 4:] == 0).all()
    assert r.span_rows == 163 and r._step_variant(192, 0) == 0 and r._step_variant(160, 0) == 256 and r._step_variant(128, 1) == 0


def test_trace_runner_program(models, tmp_path):
    """bin/trace_run as a user calls it (reference ops on the CPU)."""
    import numpy as np

    path, doc, w = models("odd", 2.0)
    toks, want = clear_choices(doc, w, 64, 20 + 4, "odd")
    lines = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:30], "want": [0, 29]}], "end": []}, {"step": 1, "entries": [{"id": "x", "tokens": toks[30:50], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": toks[50:51], "want": [0]}], "end": ["x"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64", "--device", "cpu"],
                       input="\n".join(json.dumps(x) for x in lines) + "\n", capture_output=True, text=True, timeout=120)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    assert not (tmp_path / "1.f32").exists()
    got = torch.from_numpy(np.concatenate([np.fromfile(tmp_path / f"{i}.f32", dtype="<f4").reshape(-1, doc["vocab"]) for i in (0, 2)]))
    close(got, want[[0, 29, 50]], "fp32")


def test_openai_server_and_command_line(models, tmp_path):
    """Chat completion over HTTP, and greedy generation on the command line."""
    import urllib.request

    from kvmini.server.native import start_native_in_thread

    eng = LLMEngine(EngineConfig(model="pipilix-tiny", device="cpu", dtype="fp32", max_num_seqs=4, max_model_len=256, max_batched_tokens=64))
    _srv, url, stop = start_native_in_thread(eng, model_name="v")
    try:
        body = json.dumps({"model": "v", "messages": [{"role": "user", "content": "hi there"}], "max_tokens": 8}).encode()
        r = json.loads(urllib.request.urlopen(urllib.request.Request(url + "/v1/chat/completions", body, {"Content-Type": "application/json"}), timeout=60).read())
        assert r["usage"]["completion_tokens"] == 8
    finally:
        stop()
    path, doc, w = models("plain")
    out = tmp_path / "o.jsonl"
    p = subprocess.run([sys.executable, "-m", "kvmini", "generate", "--model", path, "--device", "cpu", "--dtype", "fp32", "--prompt", "hello there", "--max-tokens", "6", "--max-model-len", "128",
                        "--out", str(out)], capture_output=True, text=True, timeout=120, cwd=ROOT)
    assert p.returncode == 0, p.stderr[-2000:]
    from kvmini.engine.tokenizer import get_tokenizer

    prompt = get_tokenizer(doc["vocab"], 1, -1).encode("hello there", add_bos=True)
    assert json.loads(out.read_text().splitlines()[0])["token_ids"] == oracle.greedy(doc, w, prompt, 6)
