"""The Gebasun design through the engine against the plain model of tests/gebasun_oracle.py: every mechanism alone, prompts,
decoding, portions, batches, re-used pages and slots, greedy generation.  Each test runs on the CPU ops, and (marked gpu) on the
HIP kernels in fp32 and bf16."""

import json
import math
import os
import subprocess
import sys

import gebasun_oracle as oracle
import pytest
import torch
from hybrid_testing import BACKENDS, ROOT, TYPES, close, feed, make_step, mixers_of, rel, replay, save, tokens

from kvmini.engine.engine import EngineConfig, LLMEngine
from kvmini.engine.replay import engine_for
from kvmini.engine.scheduler import SamplingParams
from kvmini.models import gebasun, hybrid, registry


# ---- configurations: sizes, layer orders and constants of their own
def att(heads, kv, dim, window, bias_max, scale=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "mask": {"size": window}, "bias_max": bias_max, "scale": dim ** -0.5 if scale is None else scale}}


def att2(heads, kv, dim, window, keep, rot, base=10000.0, scale=None):
    return {"type": "attention_2", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "mask": {"size": window, "keep_first": keep}, "rot": {"base": base, "dims": rot},
                                             "scale": dim ** -0.5 if scale is None else scale}}


def ssm(heads, vdim, state, groups, conv, norm_groups):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}}


def moe(la, experts, top, ff, shared):
    m = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    return dict(la, mlp=dict(m, shared={"ff": shared}) if shared else m)


def bare(la):
    return dict(la, mlp=None)


CONFIGS = {
    # odd sizes everywhere, a state space first, layers without a feed-forward (also in front of one with), a mixture without a shared expert,
    # parts of a norm that are not whole heads
    "odd": dict(vocab=131, width=75, norm={"eps": 1e-3},
                layers=[moe(ssm(3, 14, 22, 1, 3, 2), 5, 2, 36, 44), bare(att2(6, 2, 20, 29, 5, 6, 300.0, 0.5)), moe(att(3, 3, 12, 21, 18, 0.8), 7, 3, 20, 0), bare(ssm(4, 10, 9, 2, 4, 1)),
                        moe(att2(5, 1, 36, 50, 17, 36, 700.0), 3, 3, 40, 28), moe(att(4, 2, 20, 45, 70, 0.4), 6, 1, 24, 30)]),
    # constants at their plain values: one head, one expert a token, one kept token, a window that the kept tokens touch, one tap, whole tiles
    "plain": dict(vocab=200, width=64, norm={"eps": 1e-6},
                  layers=[moe(att2(1, 1, 64, 32, 1, 64), 4, 1, 64, 64), moe(ssm(1, 64, 64, 1, 1, 1), 4, 2, 64, 64), moe(att(1, 1, 64, 64, 64), 4, 4, 64, 64), moe(att2(2, 2, 32, 16, 16, 32), 2, 1, 64, 64)]),
    # large heads and states, many experts chosen, many query heads per key head, a window beyond the request, wide convolution
    "wide": dict(vocab=97, width=140, norm={"eps": 1e-4},
                 layers=[moe(att2(4, 2, 130, 40, 33, 40, 500000.0, 0.1), 20, 6, 44, 90), moe(ssm(2, 144, 200, 2, 6, 4), 3, 2, 60, 30), moe(att(17, 1, 24, 3000, 200, 0.4), 70, 3, 24, 130),
                         bare(ssm(6, 24, 140, 3, 2, 6))]),
    # sizes past the matrix-core kernels (heads above 256), no rotation, no kept token, a window of one
    "huge": dict(vocab=83, width=48, norm={"eps": 1e-5},
                 layers=[moe(att2(2, 1, 300, 20, 3, 8), 5, 2, 24, 20), moe(ssm(2, 280, 12, 1, 4, 5), 4, 1, 16, 16), bare(att2(2, 2, 16, 1, 0, 0)), moe(att(2, 1, 264, 37, 30, 0.1), 4, 2, 24, 24)]),
    # contexts that decode steps share out over many workgroups
    "long": dict(vocab=83, width=48, norm={"eps": 1e-6},
                 layers=[bare(att2(2, 1, 16, 1000, 40, 8, 500.0, 1.0)), bare(ssm(2, 16, 24, 1, 4, 2)), bare(att(3, 1, 24, 700, 600, 0.8))]),
}


def make_model(name, seed=0):
    """(config.json document, weights as float64 that are exact in bf16).  Decays reach from a few tokens to hundreds."""
    doc = dict(CONFIGS[name], architecture="Gebasun")
    gen = torch.Generator().manual_seed(seed)
    w = {}
    for n, s in hybrid.tensor_shapes(gebasun.config_from_json(doc)).items():
        r = torch.randn(s, generator=gen, dtype=torch.float64)
        leaf = n.rsplit(".", 1)[-1]
        if leaf.startswith("norm"):
            r = 1 + 0.2 * r
        elif n == "embed":
            r = r * 2.0
        elif leaf == "A_log":
            r = r - 1.5
        elif leaf == "dt_bias":
            r = r - 2.0
        elif leaf == "b":
            r = 0.3 * r
        elif leaf == "rel":
            r = 1.5 * r
        elif leaf not in ("D", "sink"):
            r = r / math.sqrt(s[-1])
        w[n] = r.to(torch.bfloat16).double()
    return doc, w


_built = {}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    def get(name):
        if name not in _built:
            doc, w = make_model(name, seed=len(name) + 5)
            _built[name] = (save(tmp_path_factory.mktemp(name), doc, w), doc, w)
        return _built[name]

    return get


_requests = {}


def clear_choices(doc, w, n, seed, key, margin=0.04):
    """(request of n tokens, the plain model's logits): random tokens, changed where a choice of experts is so close that rounding could
    turn it (what follows would be another computation)."""
    key = (key, n, seed)
    if key not in _requests:
        toks, upto, i = tokens(n, doc["vocab"], seed), min(n, 16), 0
        while True:  # (a growing prefix: what comes later does not matter to it)
            tight = (oracle.closest_choices(doc, w, toks[:upto]) < margin).nonzero().view(-1)
            if len(tight):
                toks[int(tight[0])] = (toks[int(tight[0])] + 1 + i) % doc["vocab"]
                i += 1
                assert i < 60 * n
            elif upto == n:
                break
            else:
                upto = min(n, upto + 16)
        _requests[key] = (toks, oracle.logits(doc, w, toks))
    return _requests[key]


def tables(n, dims, base, device):
    """cos / sin of the angles, [positions, dims / 2]."""
    a = torch.arange(n, dtype=torch.float64)[:, None] * base ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / max(1, dims))
    return a.cos().float().to(device), a.sin().float().to(device)


def sections(parts):
    """(columns [T, n], first column of each part): the parts side by side, each from a multiple of eight on."""
    parts = [torch.nn.functional.pad(p, (0, -p.shape[1] % 8)) for p in parts]
    return torch.cat(parts, 1), [0, *torch.tensor([p.shape[1] for p in parts]).cumsum(0).tolist()]


def through_portions(mx, proj, width, t, device, ty, run, slots, per=24):
    """Two sequences of t tokens in portions side by side (cut inside and at the edges of pages and chunks), then token by token:
    [2, t, width] of what ``run(rows, out, step)`` writes behind eight columns that it must leave alone."""
    got, at = torch.zeros(2, t, width, dtype=torch.float64), [0, 0]
    for n in [(70, 1), (37, 30), (2, 1), (1, 129), (150, 2), (3, 1), (2, 100), (55, 0), (0, 57)] + [(1, 1)] * 9 + [(1, 0)]:
        ps = [(x, at[i], slots[i]) for i, x in enumerate(n) if x]
        st = make_step(mx, ps, device, n_blocks=160, per=per, long=at[0] % 2 == 1)
        rows = torch.cat([torch.arange(p0, p0 + x) for x, p0, _ in ps])
        x = torch.full((st.rows, proj.shape[1]), float("nan"), dtype=ty, device=device)
        x[: len(rows)] = proj[rows.to(device)]
        out = torch.zeros(st.rows, 8 + width, dtype=ty, device=device)
        run(x, out, st)
        assert bool((out[:, :8] == 0).all())
        r = 0
        for i, z in enumerate(n):
            got[i, at[i] : at[i] + z] = out[r : r + z, 8:].double().cpu()
            r += z
            at[i] += z
    assert at == [t, t]
    return got


# ---- mechanisms alone ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width,t", [(75, 19), (300, 5), (2048, 130), (4500, 19), (4096, 140)])
def test_one_update_with_both_results_alone(backend, width, t):
    device, dtype = backend
    ty, mx = TYPES[dtype], mixers_of(device)
    ld, eps, top = hybrid.pad_k(width), 1e-3, 3
    gen = torch.Generator().manual_seed(width)
    rnd = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()  # noqa: E731
    p32 = lambda v: torch.nn.functional.pad(v, (0, ld - width)).float().contiguous().to(device)  # noqa: E731
    x0, y, y2, bias, g, g2 = rnd(t, width), rnd(t, width), rnd(t, width), rnd(width), 1 + 0.2 * rnd(width), 1 + 0.2 * rnd(width)

    def check(more, new, two=True):
        x = p32(x0)
        a, b = mx.parallel_residual(x, *more, p32(g), p32(g2) if two else None, eps, width, ty)
        unit, tol = oracle.rms_unit(new, eps), 4e-6 if dtype == "fp32" else 4e-3
        assert rel(x[:, :width], new) < 2e-6 and rel(a[:, :width], unit * g) < tol and bool((x[:, width:] == 0).all()) and bool((a[:, width:] == 0).all())
        assert (b is not None) == two
        if two:
            assert rel(b[:, :width], unit * g2) < tol and bool((b[:, width:] == 0).all())

    check((None, None, None), x0)
    check((p32(y).to(ty), None, None), x0 + y)
    check((p32(y).to(ty), p32(bias), None), x0 + y + bias, two=False)
    if device == "cpu":
        check((p32(y), p32(bias), p32(y2)), x0 + y + bias + y2)
        return
    # split sums, and experts' rows (weight zero: the row was never written) beside a shared expert's
    from kvmini.ops.hip_ops import Partial

    slabs = torch.stack([p32(rnd(t, width)) for _ in range(3)])
    total = slabs.double().sum(0)[:, :width].cpu()
    rows, wt, sh = rnd(t * top, width), torch.rand(t, top, generator=gen), rnd(t, width)
    wt[2, 1], wt[4] = 0, 0
    dev = p32(rows).to(ty)
    dev[wt.view(-1).to(device) == 0] = float("nan")
    mixed = (rows.view(t, top, width) * wt.double()[:, :, None]).sum(1)
    check((Partial(slabs), p32(bias), mx.ExpertRows(dev, wt.to(device))), x0 + total + bias + mixed)
    check((p32(y).to(ty), None, mx.ExpertRows(dev, wt.to(device), p32(sh).to(ty))), x0 + y + mixed + sh, two=False)
    check((Partial(slabs), None, mx.ExpertRows(dev, wt.to(device), Partial(slabs))), x0 + 2 * total + mixed)


def test_distance_buckets():
    """Against the plain rule, and its landmarks: one row each for near distances, the last one from the largest distance on."""
    for buckets, longest in ((32, 128), (32, 120), (12, 30), (8, 5), (2, 64), (64, 5000), (16, 9), (16, 128)):
        rows = hybrid.distance_buckets(buckets, longest, longest + 300)
        assert rows == [oracle.distance_bucket(n, buckets, longest) for n in range(longest + 300)]
        assert rows[: buckets // 2] == list(range(buckets // 2)) and rows[longest:] == [buckets - 1] * 300 and sorted(rows) == rows and max(rows) == buckets - 1
    assert hybrid.distance_buckets(8, 4, 8) == [0, 1, 2, 3, 7, 7, 7, 7]
    assert [hybrid.distance_buckets(16, 128, 129)[n] for n in (8, 11, 12, 15, 16, 32, 64, 127, 128)] == [8, 8, 9, 9, 10, 12, 14, 15, 15]


WINDOWED = [("attention", 3, 3, 20, 29, 0, 0, 12, 18), ("attention", 8, 2, 64, 64, 0, 0, 32, 128), ("attention", 4, 2, 128, 100, 0, 0, 16, 80), ("attention", 17, 1, 40, 45, 0, 0, 8, 400), ("attention", 2, 1, 130, 33, 0, 0, 4, 9),
            ("attention", 2, 2, 300, 17, 0, 0, 6, 40), ("attention", 6, 2, 96, 1000, 0, 0, 32, 250), ("attention", 5, 1, 56, 1, 0, 0, 2, 64),
            ("attention_2", 6, 2, 20, 29, 5, 6, 0, 0), ("attention_2", 2, 1, 64, 32, 1, 64, 0, 0), ("attention_2", 8, 2, 128, 100, 33, 32, 0, 0), ("attention_2", 33, 1, 40, 45, 64, 38, 0, 0), ("attention_2", 2, 2, 200, 64, 16, 96, 0, 0),
            ("attention_2", 2, 1, 300, 20, 3, 8, 0, 0), ("attention_2", 4, 4, 96, 70, 100, 0, 0, 0), ("attention_2", 3, 1, 72, 16, 0, 48, 0, 0), ("attention_2", 4, 2, 64, 1000, 7, 16, 0, 0)]


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("kind,heads,kv,dim,window,keep,rot,buckets,longest", WINDOWED)
def test_windowed_attention_alone(backend, kind, heads, kv, dim, window, keep, rot, buckets, longest):
    """One branch over a prompt in portions beside another sequence's, then single tokens.  For some queries one key stands out: the first and
    the last inside the window, the first ones just outside, the last kept token and the one behind it, page borders, the first tokens, the
    query's own; for others the sink takes nearly all."""
    device, dtype = backend
    ty, mx, t, eps, base = TYPES[dtype], mixers_of(device), 330, 1e-5, 700.0
    two = kind == "attention_2"
    gen = torch.Generator().manual_seed(dim + window + keep)
    rnd = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()  # noqa: E731
    q, k, bq, bk, gl = rnd(t, heads, dim), rnd(t, kv, dim), 0.5 * rnd(heads, dim), 0.5 * rnd(kv, dim), rnd(t, heads * dim)
    rel_table = 2.0 * rnd(max(buckets, 2), heads)
    sink = rnd(heads)
    sink[0] = 5.0
    scale, group = 3.0 / math.sqrt(dim), [h // (heads // kv) for h in range(heads)]
    places = {"edge": lambda i: i - window + 1, "out": lambda i: i - window, "further out": lambda i: i - window - 1, "kept": lambda i: keep - 1, "not kept": lambda i: keep, "own": lambda i: i, "first": lambda i: 0,
              "page": lambda i: (i // 16) * 16, "before page": lambda i: (i // 16) * 16 - 1, "half": lambda i: i - (window + 1) // 2, "step": lambda i: i - window + 32}
    shown = {n: 0 for n in places}
    for i in range(t):
        name = list(places)[(i * 7 + i // 16) % len(places)] if i % 3 else None
        j = places[name](i) if name else -1
        if not 0 <= j <= i:
            continue
        shown[name] += 1
        a = k[j] + bk
        if two and rot:  # before its own rotation, what turns into the key's direction
            a = oracle.rotate_halves(a[None], rot, base, first=j - i)[0]
        q[i] = a[group] - bq
    q = q.to(torch.bfloat16).double()
    assert all(shown[n] for n in places if n not in ("kept", "not kept") and (n != "step" or window >= 32)) or window >= t
    qt, kt, v = q + bq, k + bk, k + bk
    if two:
        qt, kt = (oracle.rotate_halves(x, rot, base) for x in (qt, kt))
    add = None if two else (lambda n: rel_table[oracle.distance_bucket(n, buckets, longest)])
    o = oracle.attend(oracle.rms_unit(qt, eps), oracle.rms_unit(kt, eps), v, scale, sink, lambda i, j: oracle.sees(i, j, window, keep), add).reshape(t, -1)
    want = o * (torch.sigmoid(gl) if two else 1.0) * 0.7
    common = dict(key_values=True, norm_gains=False, sink=True)
    m = hybrid.AttentionSpec(heads, kv, dim, dim, scale, 0, base, rot, window, keep, "element", out_bias=False, **common) if two else \
        hybrid.AttentionSpec(heads, kv, dim, dim, scale, window=window, gate="none", rel=True, rel_max=longest, rel_buckets=buckets, **common)
    proj, off = sections([q.reshape(t, -1), k.reshape(t, -1)] + ([gl] if two else []))
    v32 = lambda x: x.float().contiguous().to(device)  # noqa: E731
    w = hybrid.AttentionWeights(off[0], off[1], off[1], off[2] if two else 0, 8, v32(torch.cat((bq.view(-1), bk.view(-1), bk.view(-1)))), torch.ones(dim, device=device), torch.ones(dim, device=device), v32(sink))
    if not two:
        w.rel = v32(torch.stack([rel_table[oracle.distance_bucket(n, buckets, longest)] for n in range(min(window, longest + 1))], 1))
    cache = tuple(torch.full((160, kv, 16, p), 3.0, dtype=ty, device=device) for p in mx.cache_pads(m, ty))  # (left over from somebody else)
    turns = tables(t + 1, rot, base, device)
    got = through_portions(mx, proj.to(ty).to(device), heads * dim, t, device, ty, lambda x, out, st: mx.attention(m, w, 0.7, eps, x, out, cache, turns, st), (1, 3))
    for i in range(2):
        each = (got[i] - want).norm(dim=1) / want.norm(dim=1)
        assert rel(got[i], want) < (4e-6 if dtype == "fp32" else 0.02), i
        assert float(each.max()) < (6e-5 if dtype == "fp32" else 0.1), (i, int(each.argmax()))


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,vdim,dim,groups,taps,parts", [(3, 14, 22, 1, 3, 2), (2, 64, 64, 1, 4, 1), (4, 64, 128, 2, 4, 4), (1, 128, 128, 1, 4, 1), (6, 32, 48, 2, 2, 3), (2, 200, 40, 2, 5, 2), (3, 20, 200, 3, 4, 1),
                                                              (1, 280, 300, 1, 1, 8), (8, 8, 16, 1, 4, 8), (4, 1, 5, 4, 4, 2), (2, 600, 16, 1, 4, 1), (32, 40, 24, 4, 8, 5)])
def test_state_space_alone(backend, heads, vdim, dim, groups, taps, parts):
    """One branch over a prompt in portions beside another sequence's, then single tokens.  Some inputs are large, so that what follows rests on
    them until they have decayed; heads forget within a token or hardly at all; some steps wipe a state; slots hold somebody else's memory."""
    device, dtype = backend
    ty, mx, t, eps = TYPES[dtype], mixers_of(device), 330, 1e-5
    m = hybrid.StateSpaceSpec(heads, vdim, dim, groups, taps, parts)
    gen = torch.Generator().manual_seed(dim + vdim)
    rnd = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()  # noqa: E731
    z, xbc, dt = rnd(t, m.inner), rnd(t, m.channels), rnd(t, heads)
    for j in (0, 1, 15, 16, 63, 64, 69, 70, 106, 107, 108, 127, 128, 200, 250, 256, 300):
        xbc[j] *= 4
    dt[40] += 30
    dt[201] += 60
    conv, conv_b, dt_b, d, norm = rnd(m.channels, taps), 0.3 * rnd(m.channels), rnd(heads) - 2, rnd(heads), 1 + 0.2 * rnd(m.inner)
    a_log = torch.linspace(-6.0, 2.5, heads, dtype=torch.float64).to(torch.bfloat16).double()
    y = oracle.silu(oracle.causal_convolution(xbc, conv, conv_b))
    if dtype == "bf16":  # (the convolution's results are the activations' type)
        y = y.to(torch.bfloat16).double()
    x, b, c = y.split([m.inner, groups * dim, groups * dim], -1)
    o = oracle.selective_sums(x.view(t, heads, vdim), b.view(t, groups, dim), c.view(t, groups, dim), oracle.softplus(dt + dt_b), a_log, d).reshape(t, -1)
    want = oracle.gated_group_norm(o, z, parts, norm, eps) * 0.7
    proj, off = sections([z, xbc, dt])
    v32 = lambda v: v.float().contiguous().to(device)  # noqa: E731
    w = hybrid.StateSpaceWeights(*off[:3], 8, v32(conv.T), v32(conv_b), v32(dt_b), v32(a_log), v32(d), v32(norm))
    state, ring = torch.zeros(5, *m.state_shape, device=device), torch.full((5, *m.ring_shape), 9.0, dtype=ty, device=device)
    state[:, :, :dim, :vdim] = 7.0
    branch = mx.StateSpace(m, w, 0.7, eps, state, ring)
    got = through_portions(mx, proj.to(ty).to(device), m.inner, t, device, ty, branch.run, (4, 1))
    assert bool((state[0] == state[2]).all()) and bool((state[:, :, dim:] == 0).all()) and bool((state[:, :, :, vdim:] == 0).all()) and bool((ring[0] == 9).all())
    for i in range(2):
        each = (got[i] - want).norm(dim=1) / want.norm(dim=1)
        assert rel(got[i], want) < (4e-6 if dtype == "fp32" else 6e-3), i
        assert float(each.max()) < (1e-4 if dtype == "fp32" else 0.03), (i, int(each.argmax()))  # (bf16: results whose rounding falls to the other side)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("experts,top,width,ff,shared,t", [(5, 2, 75, 36, 50, 20), (16, 1, 128, 64, 64, 1), (70, 6, 300, 100, 0, 77), (3, 3, 256, 40, 300, 128), (64, 4, 140, 72, 130, 200), (8, 4, 256, 96, 30, 333),
                                                           (300, 8, 64, 24, 40, 150), (1, 1, 64, 200, 20, 140), (79, 5, 64, 40, 24, 33)])
def test_squared_relu_experts_by_the_chosen_logits_alone(backend, experts, top, width, ff, shared, t):
    """Padding rows in between choose nobody."""
    device, dtype = backend
    ty, mx = TYPES[dtype], mixers_of(device)
    gen = torch.Generator().manual_seed(experts + ff)
    rnd = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()  # noqa: E731
    spec = hybrid.MoeSpec(experts, top, ff, scores="chosen", correction=False, act="relu2", shared_ff=shared, shared_gate=False, bias=True)
    cfg = hybrid.HybridConfig("m", 8, width, (hybrid.LayerSpec((hybrid.BranchSpec(hybrid.StateSpaceSpec(1, 8, 8, 1, 2), "mix"),), moe=spec),), 1e-5, wiring="parallel")
    shapes = hybrid.tensor_shapes(cfg)
    w = {"m." + n[len("l0.mlp.") :]: (2 * rnd(*s) / math.sqrt(s[-1])).to(torch.bfloat16).double() for n, s in shapes.items() if n.startswith("l0.mlp.")}
    w["m.router.b"] = 2 * rnd(experts)  # (it turns choices)
    assert "m.e0.gate" not in w and "m.shared.sg" not in w and ("m.shared.up" in w) == (shared > 0)
    h = rnd(4 * t + 64, width)  # (rows with a clear choice)
    h = h[(oracle.choice_margin(h @ w["m.router"].T + w["m.router.b"], top) > 1e-4).nonzero().view(-1)][:t]
    assert len(h) == t
    want = oracle.mixture(h, w, "m", {"router": {"top": top, "experts": experts}, "shared": {"ff": shared} if shared else None})
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
    y = mx.experts(spec, mw, x.to(ty).to(device), st)
    if device != "cpu":
        dead = torch.ones(rows, dtype=torch.bool)
        dead[live] = False
        assert bool((y.weights[dead.to(device)] == 0).all()) and (y.shared is not None) == (shared > 0) and y.shared_gate is None
        assert float((y.weights[live.to(device)].sum(1) - 1).abs().max()) < 1e-6
        clean = torch.where(y.weights.view(-1, 1) == 0, torch.zeros_like(y.rows.float()), y.rows.float())
        total = (clean.view(rows, top, -1) * y.weights[:, :, None]).sum(1)
        if shared:
            total = total + (y.shared.slabs.sum(0) if hasattr(y.shared, "slabs") else y.shared)[:rows, : cfg.ld].float()
        y = total
    assert rel(y[live.to(device), :width], want) < (3e-6 if dtype == "fp32" else 0.012)
    assert bool((y[live.to(device), width:] == 0).all())


# ---- the whole model ----------------------------------------------------------------------------------------------
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["odd", "plain", "wide", "huge"])
def test_stream_after_every_layer(backend, name, models):
    path, doc, w = models(name)
    toks, _ = clear_choices(doc, w, 45, 3, name)
    rp = replay(path, backend)
    got = []
    rp.engine.runner._after_layer = lambda ri, x: got.append(x[: len(toks), : doc["width"]].double().cpu().clone())
    rp.step([{"id": 0, "tokens": toks, "want": [0]}], [0])
    want = oracle.layer_outputs(doc, w, toks)
    assert len(got) == len(want) == len(rp.engine.mcfg.runs)
    for ri, (a, b) in enumerate(zip(got, want)):
        assert rel(a, b) < (1e-5 if backend[1] == "fp32" else 0.02), ri


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", [n for n in CONFIGS if n != "long"])
def test_prompts_portions_and_decoding_agree_with_the_plain_model(backend, name, models):
    """One request whole, in portions of changing size (down to two tokens, cut in the middle of pages, windows and chunks), and token by
    token: the same logits everywhere."""
    path, doc, w = models(name)
    toks, want = clear_choices(doc, w, 146, 7, name)
    rp = replay(path, backend)
    for plan in ([146], [2, 3, 17, 2, 30, 5, 2, 85], [110] + [1] * 36, [1] * 146, [33, 1, 2, 1, 66, 43], [64, 64, 18], [65, 63, 2, 16]):
        got = feed(rp, [[(0, n)] for n in plan], {0: toks})[0]
        close(got, want, backend[1], (name, plan))


@pytest.mark.parametrize("backend", BACKENDS)
def test_batches_of_unequal_requests_and_reused_pages_and_slots(backend, models):
    """Up to four live requests, portions beside single tokens, in a pool that just holds them; pages and slots of finished requests
    go to new ones.  Each request's logits are those of the request alone."""
    path, doc, w = models("odd")
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
    """Decoding across many pages, windows and chunks, one token a step."""
    path, doc, w = models("plain")
    toks, want = clear_choices(doc, w, 150, 9, "plain")
    got = feed(replay(path, backend, graphs=True), [[(0, 6)]] + [[(0, 1)]] * 144, {0: toks})[0]
    close(got, want, backend[1])


@pytest.mark.parametrize("backend", BACKENDS[:2])
def test_greedy_generation_through_the_scheduler(backend, models):
    """The engine's own entry point: prompts longer than a step's budget, more requests than slots, launch-ahead stepping, and a pool
    so small that sequences are preempted and start over — the plain model's greedy continuations."""
    device, dtype = backend
    path, doc, w = models("odd")
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
        assert eng.bm.prefix_hits == 0  # (a recurrent state cannot be taken over)
    hot = SamplingParams(max_tokens=n_new, temperature=0.8, top_k=20, seed=5)
    out = eng.generate(prompts, hot)
    assert out == eng.generate(prompts, hot) and all(0 <= t < doc["vocab"] for o in out for t in o)


@pytest.mark.gpu
@pytest.mark.parametrize("name", ["odd", "plain"])
def test_replayed_graphs_equal_eager_steps(models, name):
    """Every step shape of a mixed schedule, replayed several times with eager work in between, against the same steps without graphs: bit
    for bit."""
    path, doc, _w = models(name)
    reqs = {i: tokens(n, doc["vocab"], 60 + i) for i, n in enumerate([70, 40, 90])}
    plan = [[(0, 20), (1, 10)], [(0, 1), (1, 1), (2, 50)], [(0, 1), (1, 1), (2, 1)], [(0, 1), (1, 1), (2, 2)], [(0, 47), (2, 1)], [(1, 2), (2, 2)], [(1, 25), (2, 34)]]
    a = replay(path, ("cuda:0", "bf16"), 256, graphs=True)
    b = replay(path, ("cuda:0", "bf16"), 256)
    assert a.engine.runner.graphs and not b.engine.runner.graphs
    for _ in range(4):
        ga, gb = feed(a, plan, reqs), feed(b, plan, reqs)
        assert all(torch.equal(ga[i], gb[i]) for i in reqs)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["bf16", "fp32"])
def test_long_contexts(models, dtype):
    """More than 2000 tokens of context, beside a short request, in prompts and in decode steps (graphs) that share the windows' keys out."""
    path, doc, w = models("long")
    reqs = {0: tokens(2112, doc["vocab"], 1), 1: tokens(40, doc["vocab"], 2)}
    rp = replay(path, ("cuda:0", dtype), 2304, graphs=True)
    rp.engine.runner.SPLIT_KV_MIN_CTX = 512
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
        n = int((oracle.closest_choices(doc, w, p + o)[len(p) :] < 0.04).long().cumsum(0).eq(0).sum())  # (up to a choice that rounding can turn)
        assert len(o) == 12 and float(gap[: n + 1].max()) < 0.1 * float(lg.std()), gap
    hot = SamplingParams(max_tokens=12, temperature=0.9, top_k=30, top_p=0.95, seed=11)
    out = eng.generate(prompts, hot)
    assert out == eng.generate(prompts, hot) and all(len(o) == 12 and 0 <= min(o) and max(o) < doc["vocab"] for o in out)


# ---- the framework around it --------------------------------------------------------------------------------------
def test_registry_and_configuration(models):
    path, doc, _w = models("odd")
    cfg, wpath = registry.resolve_model(path)
    assert cfg.family == "gebasun" and wpath == path and cfg.recurrent and cfg.num_layers == 6 and cfg.wiring == "parallel" and cfg.rms_eps == 1e-3
    assert cfg.layers[0].branches[0].mixer == hybrid.StateSpaceSpec(3, 14, 22, 1, 3, 2)
    common = dict(key_values=True, norm_gains=False, sink=True)
    assert cfg.layers[1].branches[0].mixer == hybrid.AttentionSpec(6, 2, 20, 20, 0.5, 0, 300.0, 6, 29, 5, "element", out_bias=False, **common)
    assert cfg.layers[2].branches[0].mixer == hybrid.AttentionSpec(3, 3, 12, 12, 0.8, window=21, gate="none", rel=True, rel_max=18, **common)
    assert cfg.layers[0].moe == hybrid.MoeSpec(5, 2, 36, scores="chosen", correction=False, act="relu2", shared_ff=44, shared_gate=False, bias=True)
    assert cfg.layers[1].moe is None and cfg.layers[2].moe.shared_ff == 0
    names = hybrid.tensor_shapes(cfg)
    assert names["l0.mix.in"] == (3 * 14 + 3 * 14 + 44 + 3, 75) and names["l0.mix.conv"] == (86, 3) and names["l1.mix.g"] == (120, 75) and names["l0.mlp.router.b"] == (5,) and names["head"] == (131, 75)
    assert not {"l1.mix.v", "l1.mix.o.b", "l1.norm2", "l2.mix.g", "l1.mix.q.norm", "l0.norm1b", "l0.mlp.e0.gate", "l0.mlp.shared.sg", "l0.mlp.correction"} & set(names) and "l2.mix.o.b" in names
    assert registry.resolve_model("gebasun-tiny")[0].name == "gebasun-tiny" and {"gebasun-1b", "gebasun-8b", "zipelix-8b"} <= set(registry.preset_names())
    for key, val, why in (("type", "something", "unknown mixer"), ("mlp", {"kind": "dense"}, "unknown feed-forward")):
        bad = json.loads(json.dumps(doc))
        bad["layers"][0][key] = val
        with pytest.raises(ValueError, match=why):
            gebasun.config_from_json(bad)
    with pytest.raises(ValueError, match="architecture"):
        gebasun.config_from_json(dict(doc, architecture="Other"))
    with pytest.raises(ValueError, match="window"):
        gebasun.config_from_json(dict(doc, layers=[bare(att(1, 1, 8, 0, 8))]))
    uneven = att(1, 1, 8, 8, 8)
    uneven["mixer"]["vdim"] = 12
    for la, why in ((uneven, "that are the keys"), (att(3, 2, 8, 8, 8), "heads"), (att2(2, 1, 8, 8, 1, 10), "rotated"), (att2(2, 1, 8, 8, -1, 8), "first tokens"), (ssm(3, 8, 8, 2, 4, 1), "heads"), (ssm(3, 8, 8, 1, 4, 5), "parts"),
                    (ssm(3, 8, 8, 1, 0, 1), "taps")):
        with pytest.raises(ValueError, match=why):
            hybrid.check_config(gebasun.config_from_json(dict(doc, layers=[bare(la)])))
    with pytest.raises(ValueError, match="experts"):
        hybrid.check_config(gebasun.config_from_json(dict(doc, layers=[moe(ssm(1, 8, 8, 1, 4, 1), 3, 4, 8, 8)])))


def test_number_of_distance_buckets_is_the_tensors(models, tmp_path):
    """The configuration does not give it: any number of rows loads, and is used."""
    _path, doc, w = models("plain")
    for rows in (6, 48, 160):  # (160: half of them is more than the largest distance)
        v = dict(w, **{"l2.mix.rel": (2 * torch.randn(rows, 1, generator=torch.Generator().manual_seed(rows))).to(torch.bfloat16).double()})
        toks = clear_choices(doc, v, 40, 3, ("rel", rows))[0]
        close(feed(replay(save(tmp_path / str(rows), doc, v), ("cpu", "fp32")), [[(0, 30)], [(0, 10)]], {0: toks})[0], oracle.logits(doc, v, toks), "fp32", rows)


def test_checkpoints_that_do_not_fit_are_refused(models, tmp_path):
    _path, doc, w = models("plain")
    short = dict(w)
    del short["l0.mix.sink"]
    with pytest.raises(KeyError, match="sink"):
        engine_for(save(tmp_path / "a", doc, short), "fp32", 64, "cpu")
    with pytest.raises(ValueError, match="shape"):
        engine_for(save(tmp_path / "b", doc, dict(w, **{"l1.mix.in": w["l1.mix.in"][:-1]})), "fp32", 64, "cpu")


def test_what_is_not_available_is_refused_by_name():
    base = dict(model="gebasun-tiny", device="cpu", dtype="fp32", max_model_len=64, max_num_seqs=2)
    for more, why in ((dict(quantization="fp8"), "quantization"), (dict(kv_cache_dtype="fp8"), "KV cache"), (dict(tp_size=2), "tensor parallelism"),
                      (dict(draft_model="tiny-draft", num_speculative_tokens=2), "speculative decoding")):
        with pytest.raises(ValueError, match=why):
            LLMEngine(EngineConfig(**base, **more))


def test_trace_runner_program(models, tmp_path):
    """bin/trace_run as a user calls it (reference ops on the CPU)."""
    import numpy as np

    path, doc, w = models("odd")
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

    eng = LLMEngine(EngineConfig(model="gebasun-tiny", device="cpu", dtype="fp32", max_num_seqs=4, max_model_len=256, max_batched_tokens=64))
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
