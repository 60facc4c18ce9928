"""The Zipelix design through the engine against the plain model of tests/zipelix_oracle.py: every mechanism alone, prompts,
decoding, portions, batches, re-used pages and slots, shared caches, greedy generation.  Each test runs on the CPU ops, and
(marked gpu) on the HIP kernels in fp32 and bf16."""

import json
import math
import os
import subprocess
import sys

import pytest
import torch
import zipelix_oracle as oracle
from hybrid_testing import BACKENDS, ROOT, TYPES, close, feed, make_step, mixers_of, rel, replay, save, tokens

from kvmini.engine.engine import EngineConfig, LLMEngine
from kvmini.engine.replay import engine_for
from kvmini.engine.scheduler import SamplingParams
from kvmini.models import hybrid, registry, zipelix


# ---- configurations: sizes, layer orders and constants of their own
def lat(heads, dim, rot, vdim, rank, base=10000.0, scale=None, src=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "rot": {"base": base, "dims": rot}, "scale": (dim + rot) ** -0.5 if scale is None else scale}
    return {"type": "latent_attention", "mixer": m if src is None else dict(m, kv_from=src)}


def ret(heads, dim, vdim, rot, decay, base=10000.0):
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "rot": {"base": base, "dims": rot}, "decay": list(decay)}}


def dense(la, ff):
    return dict(la, mlp={"kind": "dense", "ff": ff})


def moe(la, experts, top, ff, shared, scale=1.0):
    m = {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale}, "expert": {"ff": ff}}
    return dict(la, mlp=dict(m, shared={"ff": shared}) if shared else m)


def bare(la):
    return dict(la, mlp=None)


CONFIGS = {
    # odd sizes everywhere, three streams, retention first, a cache read by two later layers, a layer without a feed-forward, a mixture
    # without a shared expert
    "odd": dict(vocab=131, width=75, norm={"eps": 1e-3}, streams=3, logit_softcap=9.0,
                layers=[moe(ret(3, 22, 13, 10, (0.9, 0.99, 1.0)), 5, 2, 36, 44, 1.7), dense(lat(3, 20, 6, 12, 28, 300.0), 100), bare(ret(2, 12, 28, 12, (0.6, 0.97))),
                        moe(lat(5, 12, 6, 20, 28, 300.0, 0.3, 1), 7, 3, 20, 0, 0.6), dense(lat(2, 36, 6, 9, 28, 300.0, src=1), 40)]),
    # constants at their plain values: one stream, one head, one expert a token, whole tiles, every layer its own cache
    "plain": dict(vocab=200, width=64, norm={"eps": 1e-6}, streams=1, logit_softcap=50.0,
                  layers=[moe(lat(1, 64, 64, 64, 128), 4, 1, 64, 64), dense(ret(1, 64, 64, 64, (0.98,)), 128), dense(lat(2, 64, 32, 64, 128), 96)]),
    # large heads and latents (beyond one tile of the kernels), more streams than the kernels are written out for, many experts chosen
    "wide": dict(vocab=97, width=140, norm={"eps": 1e-4}, streams=6, logit_softcap=4.0,
                 layers=[moe(lat(2, 130, 40, 70, 300, 500000.0, 0.06), 20, 6, 44, 90, 2.5), dense(ret(2, 144, 200, 96, (0.995, 0.95), 1000.0), 40), moe(lat(17, 24, 40, 160, 300, 500000.0, 0.1, 0), 3, 3, 60, 30)]),
    # sizes past the matrix-core kernels (heads above 256, rotated parts above 64, values of retention above 256)
    "huge": dict(vocab=83, width=48, norm={"eps": 1e-5}, streams=2, logit_softcap=15.0,
                 layers=[dense(lat(2, 300, 10, 20, 96), 40), moe(ret(1, 280, 300, 128, (0.99,)), 70, 4, 24, 20), dense(lat(2, 24, 100, 40, 60, 50.0), 24), dense(lat(3, 16, 10, 30, 96, src=0), 24)]),
    # contexts that decode steps share out over many workgroups
    "long": dict(vocab=83, width=48, norm={"eps": 1e-6}, streams=4, logit_softcap=30.0, layers=[dense(lat(2, 16, 8, 24, 40), 40), dense(ret(2, 16, 24, 8, (0.999, 0.99)), 40), bare(lat(3, 24, 8, 16, 40, src=0))]),
}


def make_model(name, seed=0, sharp=1.0):
    """(config.json document, weights as float64 that are exact in bf16).  ``sharp`` scales the queries of attention, so that single keys
    dominate their softmax."""
    doc = dict(CONFIGS[name], architecture="Zipelix")
    gen = torch.Generator().manual_seed(seed)
    w = {}
    for n, s in hybrid.tensor_shapes(zipelix.config_from_json(doc)).items():
        r = torch.randn(s, generator=gen, dtype=torch.float64)
        leaf = n.rsplit(".", 1)[-1]
        if leaf.startswith("norm"):
            r = 1 + 0.2 * r
        elif ".hc" in n:
            r = 0.2 * r + (1.0 / doc["streams"] if leaf == "in" else 1.0 if leaf == "out" else 0.9 * torch.eye(doc["streams"], dtype=torch.float64))
        elif n == "embed":
            r = r * 2.0
        else:
            attends = n.endswith("mix.q") and doc["layers"][int(n[1 : n.index(".")])]["type"] == "latent_attention"
            r = r / math.sqrt(s[1]) * (sharp if attends else 1.0)
        w[n] = r.to(torch.bfloat16).double()
    return doc, w


_built = {}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    def get(name, sharp=1.0):
        key = (name, sharp)
        if key not in _built:
            doc, w = make_model(name, seed=len(name) + 5, sharp=sharp)
            _built[key] = (save(tmp_path_factory.mktemp(name), doc, w), doc, w)
        return _built[key]

    return get


_requests = {}


def clear_choices(doc, w, n, seed, key, margin=0.04):
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


def tables(n, dims, base, device):
    """cos / sin of the angles, [positions, dims / 2]."""
    a = torch.arange(n, dtype=torch.float64)[:, None] * base ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / max(1, dims))
    return a.cos().float().to(device), a.sin().float().to(device)


def sections(parts):
    """(columns [T, n], first column of each part): the parts side by side, each from a multiple of eight on."""
    parts = [torch.nn.functional.pad(p, (0, -p.shape[1] % 8)) for p in parts]
    return torch.cat(parts, 1), [0, *torch.tensor([p.shape[1] for p in parts]).cumsum(0).tolist()]


# ---- mechanisms alone ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("streams", [1, 2, 3, 4, 5, 16])
@pytest.mark.parametrize("width", [75, 300, 2048, 4500])
def test_residual_update_between_streams_alone(backend, streams, width):
    device, dtype = backend
    ty, mx = TYPES[dtype], mixers_of(device)
    ld, t, eps, top = hybrid.pad_k(width), 19, 1e-3, 3
    gen = torch.Generator().manual_seed(width + streams)
    rnd = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()  # noqa: E731
    p32 = lambda v: torch.nn.functional.pad(v, (0, ld - width)).float().contiguous().to(device)  # noqa: E731
    v32 = lambda v: v.float().to(device)  # noqa: E731
    w = {"hc.in": rnd(streams), "hc.out": rnd(streams), "hc.mix": rnd(streams, streams)}
    h = hybrid.HyperWeights(v32(w["hc.in"]), v32(w["hc.out"]), v32(w["hc.mix"]))
    g, read, e, y = 1 + 0.2 * rnd(width), rnd(streams), rnd(t, width), rnd(t, width)
    tol = 4e-6 if dtype == "fp32" else 4e-3
    x, xb = mx.split_streams(p32(e), streams, h.read, p32(g), eps, width, ty)
    old = e[None].repeat(streams, 1, 1)
    assert torch.equal(x, p32(e)[:, None].expand(t, streams, ld)) and rel(xb[:, :width], oracle.rms_unit(oracle.read_streams(old, w, "hc"), eps) * g) < tol
    old = rnd(streams, t, width)  # (streams that have come apart)

    def check(y_dev, y_true):
        x = p32(old.transpose(0, 1))
        xb = mx.hyper_residual(x, y_dev, h, v32(read), p32(g), eps, width, ty)
        new = oracle.write_streams(old, y_true, w, "hc")
        assert rel(x[:, :, :width], new.transpose(0, 1)) < 2e-6 and bool((x[:, :, width:] == 0).all()) and bool((xb[:, width:] == 0).all())
        assert rel(xb[:, :width], oracle.rms_unit(oracle.read_streams(new, {"r.in": read}, "r"), eps) * g) < tol
        assert torch.equal(mx.all_streams(streams, torch.device(device)).cpu(), torch.ones(streams))

    check(p32(y).to(ty), y)
    if device != "cpu":  # split sums, and experts' rows (weight zero: the row was never written) beside a shared expert's
        from kvmini.ops.hip_ops import Partial

        slabs = torch.stack([p32(rnd(t, width)) for _ in range(3)])
        check(Partial(slabs), slabs.double().sum(0)[:, :width].cpu())
        rows, wt, sg, sh = rnd(t * top, width), torch.rand(t, top, generator=gen), torch.rand(t, generator=gen), rnd(t, width)
        wt[2, 1], wt[5] = 0, 0
        dev = p32(rows).to(ty)
        dev[wt.view(-1).to(device) == 0] = float("nan")
        true = (rows.view(t, top, width) * wt.double()[:, :, None]).sum(1)
        check(mx.ExpertRows(dev, wt.to(device)), true)
        check(mx.ExpertRows(dev, wt.to(device), p32(sh).to(ty), sg.to(device)), true + sg.double()[:, None] * sh)
        check(mx.ExpertRows(dev, wt.to(device), Partial(slabs), sg.to(device)), true + sg.double()[:, None] * slabs.double().sum(0)[:, :width].cpu())


@pytest.mark.parametrize("backend", BACKENDS)
def test_soft_cap_alone(backend):
    device, dtype = backend
    z = torch.linspace(-60, 60, 3 * 1001, dtype=torch.float64).to(torch.bfloat16).double().view(3, 1001)
    for cap in (30.0, 2.5):
        out = torch.nn.functional.pad(z, (0, 23)).to(TYPES[dtype]).to(device)
        mixers_of(device).softcap(out[:, :1001], cap)
        assert float((out[:, :1001].double().cpu() - oracle.capped(z, cap)).abs().max()) < cap * (1e-6 if dtype == "fp32" else 4e-3) and bool((out[:, 1001:] == 0).all())


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,dim,rot,vdim,rank", [(3, 24, 6, 20, 40), (2, 128, 64, 128, 512), (17, 16, 10, 8, 200), (5, 100, 2, 130, 300), (2, 64, 64, 64, 128), (1, 200, 34, 256, 512),
                                                     (33, 40, 62, 72, 130), (2, 300, 12, 20, 96), (3, 20, 66, 12, 48), (1, 24, 8, 40, 600)])
def test_latent_attention_with_rotated_keys_alone(backend, heads, dim, rot, vdim, rank):
    """A latent branch over a prompt in portions beside another sequence's, then single tokens, and a second branch with other heads that
    reads the first one's cache.  For some queries one key is made to stand out, by its latent or by its rotated part alone: far back, at
    page borders, the first tokens, the query's own."""
    device, dtype = backend
    ty, mx, t, eps, base = TYPES[dtype], mixers_of(device), 330, 1e-5, 700.0
    gen = torch.Generator().manual_seed(dim + vdim + rank)
    rnd = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()  # noqa: E731
    c, kr, cn = rnd(t, rank), rnd(t, rot), 1 + 0.2 * rnd(rank)
    latent, turned = oracle.rms_unit(c, eps) * cn, oracle.rotate_neighbours(kr[:, None], rot, base)[:, 0]
    turns = tables(t + 1, rot, base, device)
    lay = registry._pack_for(device, ty, "auto")
    spec = lambda nh, src: hybrid.LatentSpec(nh, dim, vdim, rank, 4.0 / math.sqrt(dim * rank), 0, rot, base, "element", src)  # noqa: E731
    row = mx.cache_pads(spec(heads, -1), ty)[0]
    cache = torch.full((128, 1, 16, row), 3.0, dtype=ty, device=device)  # (left over from somebody else)
    pad = lambda x, n: torch.nn.functional.pad(x, (0, n - x.shape[-1]))  # noqa: E731
    branches = []
    for nh, src in ((heads, -1), (heads + 1, 0)):
        m = spec(nh, src)
        uk, uv = rnd(nh * dim, rank), (rnd(nh * vdim, rank) / math.sqrt(rank)).to(torch.bfloat16).double()
        k = torch.cat(((latent @ uk.T).view(t, nh, dim), turned[:, None].expand(t, nh, rot) * math.sqrt(rank)), -1)
        q, gl = rnd(t, nh, dim + rot), rnd(t, nh * vdim)
        for i in list(range(0, 60, 7)) + [95, 111, 127, 128, 129, 150, 200, 255, 256, 300, 323, 325, 327, 329]:
            for j in (0, 1, 2, i // 2, (i // 16) * 16, (i // 16) * 16 - 1, i):
                if 0 <= j <= i and (i + j) % 3 == 0:
                    a = k[j, :, :dim]
                    q[i, :, :dim] = a / a.pow(2).mean().sqrt()
                if 0 <= j <= i and (i + j) % 4 == 1:  # before its own rotation, what turns into the key's direction
                    back = -float(i)
                    ang = torch.tensor([back * base ** (-2.0 * x / rot) for x in range(rot // 2)], dtype=torch.float64)
                    u, v = turned[j][0::2], turned[j][1::2]
                    q[i, :, dim:] = 6 * torch.stack((u * ang.cos() - v * ang.sin(), v * ang.cos() + u * ang.sin()), -1).flatten()
        q[..., dim:] *= math.sqrt(rank)  # (rotated parts weigh as much as the others)
        q = q.to(torch.bfloat16).double()
        k = torch.cat((k[..., :dim], turned[:, None].expand(t, nh, rot)), -1)
        qt = torch.cat((q[..., :dim], oracle.rotate_neighbours(q[..., dim:], rot, base)), -1)
        want = oracle.causal_softmax_attention(qt, k, (latent @ uv.T).view(t, nh, vdim), m.scale).reshape(t, -1) * torch.sigmoid(gl) * 0.7
        dkp, dvp, rkp = lay.latent_pads(m)
        rtp = lay.rot_pad(m)
        assert row == rkp + rtp
        own = [pad(c, rkp), pad(kr, rtp)] if src < 0 else []
        proj, at = sections([pad(q[..., :dim], dkp).reshape(t, -1), pad(q[..., dim:], rtp).reshape(t, -1), *own, gl])
        ukp = torch.nn.functional.pad(uk.view(nh, dim, rank), (0, rkp - rank, 0, dkp - dim)).to(ty).to(device)
        uvp = torch.nn.functional.pad(uv.view(nh, vdim, rank), (0, rkp - rank, 0, dvp - vdim)).to(ty).to(device)
        w = hybrid.LatentWeights(at[0], at[2] if own else 0, at[2 + len(own)], 8, dkp, dvp, rkp, pad(cn, rkp).float().to(device) if own else torch.zeros(0, device=device),
                                 lay.heads(ukp.transpose(1, 2).contiguous(), m), lay.heads(uvp, m), lay(torch.cat((ukp.reshape(-1, rkp), uvp.reshape(-1, rkp)))) if lay.expands(m) else None,
                                 at[1], rtp, at[3] if own else 0)
        branches.append((m, w, proj.to(ty).to(device), want, torch.zeros(2, t, nh * vdim, dtype=torch.float64)))
    at = [0, 0]
    for n in [(70, 1), (37, 30), (2, 1), (1, 129), (150, 2), (3, 1), (2, 100), (55, 0), (0, 57)] + [(1, 1)] * 9 + [(1, 0)]:
        ps = [(x, at[i], (1, 3)[i]) for i, x in enumerate(n) if x]
        st = make_step(mx, ps, device, n_blocks=128, long=at[0] % 2 == 1, reach=t, per=24)
        rows = torch.cat([torch.arange(p0, p0 + x) for x, p0, _ in ps])
        for m, w, proj, _want, got in branches:
            x = torch.zeros(st.rows, proj.shape[1], dtype=ty, device=device)
            x[: len(rows)] = proj[rows.to(device)]
            out = torch.zeros(st.rows, 8 + m.heads * vdim, dtype=ty, device=device)
            mx.latent_attention(m, w, 0.7, eps, x, out, cache, st, turns)
            r = 0
            for i, z in enumerate(n):
                got[i, at[i] : at[i] + z] = out[r : r + z, 8:].double().cpu()
                r += z
        at = [a + z for a, z in zip(at, n)]
    assert at == [t, t]
    for b, (_m, _w, _p, want, got) in enumerate(branches):
        for i in range(2):
            each = (got[i] - want).norm(dim=1) / want.norm(dim=1)
            assert rel(got[i], want) < (4e-6 if dtype == "fp32" else 0.025), (b, i)
            assert float(each.max()) < (6e-5 if dtype == "fp32" else 0.1), (b, i, int(each.argmax()))


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("heads,dim,vdim,rot,decay", [(3, 22, 13, 10, (0.9, 0.99, 1.0)), (2, 64, 64, 64, (0.97, 0.999)), (1, 128, 128, 128, (0.995,)), (2, 40, 200, 32, (0.5, 0.98)), (2, 200, 72, 2, (0.0, 0.99)),
                                                      (1, 300, 256, 300, (0.99,)), (2, 48, 280, 16, (0.97, 1.0)), (1, 16, 1, 0, (0.9,)), (5, 132, 20, 66, (0.9, 0.92, 0.94, 0.96, 0.98))])
def test_retention_alone(backend, heads, dim, vdim, rot, decay):
    """One branch over a prompt in portions (cut inside and at the edges of the kernels' chunks) beside another sequence's, then single
    tokens.  Some keys are large, so that what follows rests on them until they have decayed; slots hold somebody else's state."""
    device, dtype = backend
    ty, mx, t, eps, base = TYPES[dtype], mixers_of(device), 330, 1e-5, 2000.0
    m = hybrid.RetentionSpec(heads, dim, vdim, decay, base, rot)
    gen = torch.Generator().manual_seed(dim + vdim)
    rnd = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()  # noqa: E731
    q, k, v, gl = rnd(t, heads, dim), rnd(t, heads, dim), rnd(t, heads, vdim), rnd(t, heads * vdim)
    for j in (0, 1, 15, 16, 63, 64, 69, 70, 106, 107, 108, 127, 128, 200, 250, 256, 300):
        k[j] *= 8
    o = oracle.decaying_sums(oracle.rotate_halves(q, rot, base), oracle.rotate_halves(k, rot, base) / math.sqrt(dim), v, list(decay))
    want = oracle.rms_unit(o, eps).reshape(t, -1) * oracle.silu(gl) * 0.7
    proj, off = sections([q.reshape(t, -1), k.reshape(t, -1), v.reshape(t, -1), gl])
    proj = proj.to(ty).to(device)
    log2 = torch.tensor([math.log2(x) if x else -1e4 for x in decay], dtype=torch.float32, device=device)
    state = torch.zeros(5, *m.state_shape, device=device)
    state[:, :, :dim, :vdim] = 7.0
    branch = mx.Retention(m, hybrid.RetentionWeights(*off[:4], 8, log2), 0.7, eps, state, tables(t, rot, base, device))
    got, at = torch.zeros(2, t, heads * vdim, dtype=torch.float64), [0, 0]
    for n in [(70, 1), (37, 30), (2, 1), (1, 129), (150, 2), (3, 1), (2, 100), (55, 0), (0, 57)] + [(1, 1)] * 9 + [(1, 0)]:
        ps = [(x, at[i], (4, 1)[i]) for i, x in enumerate(n) if x]
        st = make_step(mx, ps, device, n_blocks=160, per=24)
        rows = torch.cat([torch.arange(p0, p0 + x) for x, p0, _ in ps])
        x = torch.full((st.rows, proj.shape[1]), float("nan"), dtype=ty, device=device)
        x[: len(rows)] = proj[rows.to(device)]
        out = torch.zeros(st.rows, 8 + heads * vdim, dtype=ty, device=device)
        branch.run(x, out, st)
        r = 0
        for i, z in enumerate(n):
            got[i, at[i] : at[i] + z] = out[r : r + z, 8:].double().cpu()
            r += z
            at[i] += z
    assert at == [t, t] and bool((state[0] == state[2]).all()) and bool((state[:, :, dim:] == 0).all()) and bool((state[:, :, :, vdim:] == 0).all())
    for i in range(2):
        each = (got[i] - want).norm(dim=1) / want.norm(dim=1)
        assert rel(got[i], want) < (4e-6 if dtype == "fp32" else 4e-3), i
        assert float(each.max()) < (1e-4 if dtype == "fp32" else 6e-3), (i, int(each.argmax()))  # (bf16: the output's rounding; all else is fp32)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("experts,top,width,ff,shared,scale,t", [(5, 2, 75, 36, 50, 1.7, 20), (16, 1, 128, 64, 64, 1.0, 1), (70, 6, 300, 100, 0, 0.5, 77), (3, 3, 256, 40, 300, 2.0, 128), (64, 4, 140, 72, 130, 1.3, 200),
                                                                 (8, 4, 256, 96, 30, 1.0, 333), (300, 8, 64, 24, 40, 3.0, 150), (1, 1, 64, 200, 20, 0.7, 140), (79, 5, 64, 40, 24, 1.0, 33)])
def test_experts_by_softmax_with_a_shared_one_alone(backend, experts, top, width, ff, shared, scale, t):
    """Padding rows in between choose nobody."""
    device, dtype = backend
    ty, mx = TYPES[dtype], mixers_of(device)
    gen = torch.Generator().manual_seed(experts + ff)
    rnd = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()  # noqa: E731
    spec = hybrid.MoeSpec(experts, top, ff, scores="softmax", scale=scale, correction=False, act="silu", shared_ff=shared)
    cfg = hybrid.HybridConfig("m", 8, width, (hybrid.LayerSpec((hybrid.BranchSpec(hybrid.LatentSpec(1, 8, 8, 8, 1.0, 4), "mix"),), moe=spec),), 1e-5, wiring="hyper", streams=1, tied_head=True)
    shapes = hybrid.tensor_shapes(cfg)
    w = {"m." + n[len("l0.mlp.") :]: (2 * rnd(*s) / math.sqrt(s[1])).to(torch.bfloat16).double() for n, s in shapes.items() if n.startswith("l0.mlp.")}
    assert ("m.shared.sg" in w) == (shared > 0)
    h = rnd(4 * t + 64, width)  # (rows with a clear choice)
    h = h[(oracle.choice_margin(h @ w["m.router"].T, top) > 1e-4).nonzero().view(-1)][:t]
    assert len(h) == t
    want = oracle.mixture(h, w, "m", {"router": {"top": top, "scale": scale}, "shared": {"ff": shared} if shared else None})
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
        assert bool((y.weights[dead.to(device)] == 0).all()) and (y.shared is not None) == (shared > 0)
        clean = torch.where(y.weights.view(-1, 1) == 0, torch.zeros_like(y.rows.float()), y.rows.float())
        total = (clean.view(rows, top, -1) * y.weights[:, :, None]).sum(1)
        if shared:
            assert bool((y.shared_gate[dead.to(device)] == 0).all())
            total = total + y.shared_gate[:, None] * (y.shared.slabs.sum(0) if hasattr(y.shared, "slabs") else y.shared)[:rows, : cfg.ld].float()
        y = total
    assert rel(y[live.to(device), :width], want) < (3e-6 if dtype == "fp32" else 0.012)
    assert bool((y[live.to(device), width:] == 0).all())


# ---- the whole model ----------------------------------------------------------------------------------------------
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["odd", "wide", "huge"])
def test_sum_of_the_streams_after_every_layer(backend, name, models):
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
    """One request whole, in portions of changing size (down to two tokens, cut in the middle of pages and chunks), and token by token:
    the same logits everywhere."""
    path, doc, w = models(name, 3.0)
    toks, want = clear_choices(doc, w, 146, 7, name)
    rp = replay(path, backend)
    for plan in ([146], [2, 3, 17, 2, 30, 5, 2, 85], [110] + [1] * 36, [1] * 146, [33, 1, 2, 1, 66, 43], [64, 64, 18], [65, 63, 2, 16]):
        got = feed(rp, [[(0, n)] for n in plan], {0: toks})[0]
        close(got, want, backend[1], (name, plan))


@pytest.mark.parametrize("backend", BACKENDS)
def test_batches_of_unequal_requests_and_reused_pages_and_slots(backend, models):
    """Up to four live requests, portions beside single tokens, in a pool that just holds them; pages and slots of finished requests
    go to new ones.  Each request's logits are those of the request alone."""
    path, doc, w = models("odd", 3.0)
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
    """Decoding across many pages and chunks, one token a step."""
    path, doc, w = models("plain", 3.0)
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
    out = eng.generate(prompts, SamplingParams(max_tokens=n_new, temperature=0.8, top_k=20, seed=5))
    assert out == eng.generate(prompts, SamplingParams(max_tokens=n_new, temperature=0.8, top_k=20, seed=5)) and all(0 <= t < doc["vocab"] for o in out for t in o)


@pytest.mark.gpu
@pytest.mark.parametrize("name", ["odd", "plain"])
def test_replayed_graphs_equal_eager_steps(models, name):
    """Every step shape of a mixed schedule — also portions deep inside their request, whose workspace is larger than the step's —
    replayed several times with eager work in between, against the same steps without graphs: bit for bit."""
    path, doc, _w = models(name)
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
def test_long_contexts(models, dtype):
    """More than 2000 tokens of context, beside a short request, in prompts and in decode steps (graphs) that share the context's keys
    out."""
    path, doc, w = models("long", 4.0)
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
    prompts = [clear_choices(doc, w, n, 80 + n, "plain-soft")[0] for n in (3, 50, 9, 30, 77)]
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
    assert cfg.family == "zipelix" and wpath == path and cfg.recurrent and cfg.num_layers == 5 and cfg.streams == 3 and cfg.tied_head and cfg.logit_softcap == 9.0
    assert cfg.layers[0].branches[0].mixer == hybrid.RetentionSpec(3, 22, 13, (0.9, 0.99, 1.0), 10000.0, 10)
    assert cfg.layers[3].branches[0].mixer == hybrid.LatentSpec(5, 12, 20, 28, 0.3, 0, 6, 300.0, "element", 1)
    assert cfg.layers[0].moe == hybrid.MoeSpec(5, 2, 36, scores="softmax", scale=1.7, correction=False, act="silu", shared_ff=44) and cfg.layers[3].moe.shared_ff == 0 and cfg.layers[2].moe is None
    names = hybrid.tensor_shapes(cfg)
    assert "head" not in names and "l3.mix.dkv" not in names and "l2.norm2" not in names and "l2.hc2.mix" not in names and names["l1.mix.dkv"] == (34, 75) and names["l0.hc1.mix"] == (3, 3)
    assert registry.resolve_model("zipelix-tiny")[0].name == "zipelix-tiny" and {"zipelix-1b", "zipelix-8b", "pipilix-8b"} <= set(registry.preset_names())
    for key, val, why in (("type", "something", "unknown mixer"), ("mlp", {"kind": "sparse"}, "unknown feed-forward")):
        bad = json.loads(json.dumps(doc))
        bad["layers"][0][key] = val
        with pytest.raises(ValueError, match=why):
            zipelix.config_from_json(bad)
    with pytest.raises(ValueError, match="architecture"):
        zipelix.config_from_json(dict(doc, architecture="Other"))
    ok, other = dense(lat(1, 8, 4, 8, 8), 8), dense(ret(1, 8, 8, 8, (0.9,)), 8)
    for layers, why in (([ok, dense(lat(1, 8, 4, 8, 12, src=0), 8)], "latents of layer 0"), ([other, dense(lat(1, 8, 4, 8, 8, src=0), 8)], "latents of layer 0"),
                        ([ok, dense(lat(1, 8, 4, 8, 8, src=1), 8)], "latents of layer 1"), ([dense(ret(2, 8, 8, 8, (0.9,)), 8)], "decays"), ([dense(ret(1, 8, 8, 8, (1.5,)), 8)], "decays"),
                        ([moe(ok, 3, 4, 8, 8)], "experts")):
        with pytest.raises(ValueError, match=why):
            hybrid.check_config(zipelix.config_from_json(dict(doc, layers=layers)))
    with pytest.raises(ValueError, match="streams"):
        hybrid.check_config(zipelix.config_from_json(dict(doc, streams=17)))


def test_layers_that_share_a_cache_have_one(models):
    """Memory and its accounting: a reading layer has no pages of its own."""
    path, _doc, _w = models("odd")
    mem = engine_for(path, "fp32", 64, "cpu").runner.memory
    pages = [m[0][0] for m in mem.runs]
    assert pages[3].data_ptr() == pages[1].data_ptr() == pages[4].data_ptr() and pages[0].shape == (4, 3, 32, 16) and pages[2].shape == (4, 2, 16, 32)
    cfg, mx = registry.resolve_model(path)[0], mixers_of("cpu")
    pads = lambda m: mx.cache_pads(m, torch.float32)  # noqa: E731
    assert mem.block_bytes(cfg, 16, torch.float32, pads) == 16 * 34 * 4 and mem.state_bytes(cfg, 4, torch.float32, pads) == 4 * 4 * (3 * 32 * 16 + 2 * 16 * 32)


def test_checkpoints_that_do_not_fit_are_refused(models, tmp_path):
    _path, doc, w = models("plain")
    short = dict(w)
    del short["l0.mlp.shared.sg"]
    with pytest.raises(KeyError, match="shared.sg"):
        engine_for(save(tmp_path / "a", doc, short), "fp32", 64, "cpu")
    with pytest.raises(ValueError, match="shape"):
        engine_for(save(tmp_path / "b", doc, dict(w, **{"l1.hc2.mix": w["l1.hc2.mix"][0]})), "fp32", 64, "cpu")


def test_what_is_not_available_is_refused_by_name():
    base = dict(model="zipelix-tiny", device="cpu", dtype="fp32", max_model_len=64, max_num_seqs=2)
    for more, why in ((dict(quantization="fp8"), "quantization"), (dict(kv_cache_dtype="fp8"), "KV cache"), (dict(tp_size=2), "tensor parallelism"),
                      (dict(draft_model="tiny-draft", num_speculative_tokens=2), "speculative decoding")):
        with pytest.raises(ValueError, match=why):
            LLMEngine(EngineConfig(**base, **more))


def test_pieces_of_portions_are_staged_for_retention():
    r = LLMEngine(EngineConfig(model="zipelix-tiny", device="cpu", dtype="fp32", max_model_len=512, max_num_seqs=4, max_batched_tokens=256)).runner
    st = torch.full((sum(n for _, n in r._off.values()) + 64,), -7, dtype=torch.int32).numpy()
    r._stage_chunks(st, [(0, 1, 40, 2), (1, 130, 100, 1), (131, 5, 0, 3), (136, 64, 7, 0)])
    at, first = r._off["chunks"][0], r._off["first_chunk"][0]
    chunks = st[at : at + 4 * r.max_chunks].reshape(4, -1)
    assert chunks[:, :5].T.tolist() == [[1, 64, 100, 1], [65, 64, 164, 1], [129, 2, 228, 1], [131, 5, 0, 3], [136, 64, 7, 0]] and (chunks[1, 5:] == 0).all()
    assert st[first : first + 4].tolist() == [0, 0, 3, 4]


def test_trace_runner_program(models, tmp_path):
    """bin/trace_run as a user calls it (reference ops on the CPU)."""
    import numpy as np

    path, doc, w = models("odd", 3.0)
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

    eng = LLMEngine(EngineConfig(model="zipelix-tiny", device="cpu", dtype="fp32", max_num_seqs=4, max_model_len=256, max_batched_tokens=64))
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
