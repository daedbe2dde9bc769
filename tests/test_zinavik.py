"""Zinavik against the plain implementation in zinavik_oracle: on the CPU in
f32, on the GPU in f32 and bf16."""

import io
import json
import os
import sys
import time
from dataclasses import replace

import numpy as np
import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import zinavik_oracle as oracle  # noqa: E402
from hybrid_helpers import (EXACT, RUNS, Bytes, close, errors,  # noqa: E402
                            feed, meta_for, one_thread, portions,  # noqa: F401
                            whole)

from gridllm_amd.config import EngineConfig  # noqa: E402
from gridllm_amd.engine import InferenceEngine  # noqa: E402
from gridllm_amd.models.hybrid import HybridModel  # noqa: E402
from gridllm_amd.models.registry import (DenseFF, HybridSpec,  # noqa: E402
                                         LayerSpec, LightningMixer, Rotary,
                                         RoutedFF, Yarn, get_spec, looped,
                                         read_zinavik, resolve_spec)
from gridllm_amd.ops import build as ops_build  # noqa: E402
from gridllm_amd.ops import hybrid as hops  # noqa: E402
from gridllm_amd.ops.hybrid import Choice, Keys  # noqa: E402
from gridllm_amd.ops.reference import Glu  # noqa: E402

YARN = {"factor": 3.0, "original": 200, "fast": 9.0, "slow": 1.5}


def left(heads=4, kv_heads=2, dim=32, vdim=24, size=37, keep=5, rot=16,
         base=3000.0, scale=0.2, scaling=YARN):
    r = {"base": base, "dims": rot}
    if scaling:
        r["scaling"] = scaling
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "scale": scale, "rot": r,
            "mask": {"size": size, "keep_first": keep}}


def right(heads=3, dim=20, vdim=28, decay=(0.5, 0.93, 0.998)):
    assert len(decay) == heads
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}


def mixer(a=None, b=None, ls=0.7, rs=1.2):
    return {"left": a or left(), "right": b or right(), "left_scale": ls,
            "right_scale": rs}


def moe(experts=6, top=2, ff=40, limit=1.3, shared=72, shared_limit=0.9):
    d = {"kind": "moe", "expert": {"ff": ff, "limit": limit},
         "router": {"experts": experts, "top": top}}
    if shared:
        d["shared"] = {"ff": shared, "limit": shared_limit}
    return d


def config(*layers, vocab=130, width=96, eps=1e-5, streams=3, scale=7.0,
           loop=None):
    d = {"architecture": "Zinavik", "vocab": vocab, "width": width,
         "norm": {"eps": eps}, "streams": streams, "embedding": {"scale": scale},
         "layers": [{"type": "parallel", "mixer": m, "mlp": f}
                    for m, f in layers]}
    if loop:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


# layers of unlike sizes, with and without a feed-forward, that need padding;
# two of them run three times. All but the last choose all their experts: with
# bf16 a close call further down would change every token behind it
FULL = config(
    (mixer(), moe(3, 3)),
    (mixer(left(3, 1, 40, 72, 100, 0, 24, 50.0, 0.3), right(
        2, 70, 16, (0.9999, 0.2)), 1.0, 1.0), None),
    (mixer(left(5, 5, 72, 40, 12, 70, 72, 1e4, 0.1, None), right(
        1, 24, 130, (0.97,)), 0.3, 2.0), moe(4, 4, 64, 2.0, 0)),
    (mixer(left(9, 3, 20, 20, 1, 3, 6), right(), 1.5, 0.4),
     moe(9, 2, 130, 0.5, 40)),
    loop=(1, 3, 3))


def weights_of(cfg, seed=0):
    return oracle.random_weights(cfg, seed)


def build(cfg, run, seed=0, slots=5, pool=0, W=None, max_seq=512):
    dev, dtype = run
    W = W or weights_of(cfg, seed)
    m = HybridModel(read_zinavik(cfg), device=dev, dtype=dtype,
                    kv_slots=slots, kv_tokens=pool, max_seq=max_seq,
                    random_init=False)
    m._assemble(lambda name: W[name].to(dev))
    return m


def tokens(n, cfg=FULL, seed=0):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


def element(run):
    return torch.float32 if run[1] == "fp32" else torch.bfloat16


# ------------------------------------------------------------ each mechanism

ONE = (mixer(), None)
ALONE = {
    "both": config(ONE),
    "left": config((mixer(rs=0.0), None)),
    "right": config((mixer(ls=0.0), None)),
    "one-head": config((mixer(left(1, 1, 64, 64), right(1, 64, 64, (0.9,))),
                        None)),
    "one-value-head": config((mixer(left(7, 1, 24, 30), rs=0.1), None)),
    "more-heads-than-a-block": config((mixer(left(22, 2, 16, 16, rot=12)),
                                       None)),
    "padded-head": config((mixer(left(4, 2, 72, 72, rot=36)), None)),
    "wide-head": config((mixer(left(2, 1, 160, 130, rot=64, scale=0.05)),
                         None)),
    "values-wider-than-keys": config((mixer(left(2, 2, 8, 100, rot=8)), None)),
    "full-rotation": config((mixer(left(rot=32, base=30.0)), None)),
    "one-pair": config((mixer(left(rot=2)), None)),
    "no-scaling": config((mixer(left(scaling=None)), None)),
    "tight-scaling": config((mixer(left(rot=32, base=9.0, scaling={
        "factor": 8.0, "original": 64, "fast": 1.1, "slow": 1.0})), None)),
    "window-of-one": config((mixer(left(size=1, keep=0)), None)),
    "window-of-a-page": config((mixer(left(size=64, keep=64)), None)),
    "kept-beyond-a-page": config((mixer(left(size=3, keep=90)), None)),
    "window-beyond-all": config((mixer(left(size=9999, keep=1)), None)),
    "kept-beyond-all": config((mixer(left(size=2, keep=9999)), None)),
    "decay-zero-and-one": config((mixer(b=right(decay=(0.0, 1.0, 1e-4))),
                                  None)),
    "wide-state": config((mixer(b=right(2, 300, 200, (0.8, 0.99))), None)),
    "experts": config((mixer(), moe(shared=0))),
    "shared": config((mixer(), moe())),
    "top-one": config((mixer(), moe(19, 1))),
    "all-experts": config((mixer(), moe(5, 5))),
    "loose-limits": config((mixer(), moe(limit=50.0, shared_limit=50.0))),
    "tight-limits": config((mixer(), moe(limit=0.1, shared_limit=0.05))),
    "one-stream": config((mixer(), moe()), streams=1),
    "two-streams": config((mixer(), moe()), streams=2),
    "five-streams": config((mixer(), moe()), streams=5),
    "twelve-streams": config((mixer(), moe()), streams=12),
    "odd-width": config((mixer(), moe()), width=75),
    "coarse-eps": config((mixer(), moe()), eps=0.05),
    "scale-of-one": config((mixer(), moe()), scale=1.0),
    "loop-of-all": config((mixer(), moe()), ONE, loop=(0, 2, 2)),
    "loop-at-end": config(ONE, (mixer(), moe(4, 4)), loop=(1, 2, 3)),
    "loop-once": config(ONE, (mixer(), moe()), loop=(0, 1, 1)),
}


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("name", sorted(ALONE))
def test_mechanism_alone(name, run):
    cfg = ALONE[name]
    m = build(cfg, run)
    ids = tokens(150, cfg)
    want, layers = oracle.forward(cfg, weights_of(cfg), ids)
    trail = []
    slot = m.cache.alloc(0)
    got = m.forward_step([(slot, ids[:130], list(range(130)))], trail=trail)
    rest = feed(m, slot, ids[130:], [5, 1])          # as decoding does it
    close(torch.cat([got.cpu(), rest]), want, run)
    close(trail[-1], layers[-1][:130], run)


@pytest.mark.parametrize("run", RUNS)
def test_all_layers(run):
    m = build(FULL, run)
    ids = tokens(200)
    trail = []
    slot = m.cache.alloc(0)
    got = m.forward_step([(slot, ids, list(range(200)))], trail=trail)
    want, layers = oracle.forward(FULL, weights_of(FULL), ids)
    assert len(trail) == len(layers) == 8
    for a, b in zip(trail, layers):
        close(a, b, run)
    close(got, want, run)


@pytest.mark.parametrize("scaling", [
    None, YARN, {"factor": 1.0, "original": 64, "fast": 32.0, "slow": 1.0},
    {"factor": 40.0, "original": 4096, "fast": 32.0, "slow": 1.0},
    {"factor": 4.0, "original": 10, "fast": 64.0, "slow": 32.0}], ids=str)
@pytest.mark.parametrize("base,dims", [(1e4, 64), (30.0, 16), (5e5, 128),
                                       (7.0, 2)])
def test_frequencies(base, dims, scaling):
    got, grow = Rotary(base, dims, scaling and Yarn(**scaling)).frequencies()
    want, factor = oracle.yarn_frequencies(base, dims, scaling)
    assert got == pytest.approx(want, rel=1e-12) and grow == factor
    if scaling and scaling["factor"] == 40.0 and dims == 128:
        # fast pairs keep their speed, slow ones lose all of it
        f = [base ** (-2 * i / dims) for i in range(dims // 2)]
        assert got[0] == f[0] and got[-1] == pytest.approx(f[-1] / 40)
        assert f[30] / 40 < got[30] < f[30]


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("dim,dims", [(20, 12), (64, 64), (128, 96), (200, 8)])
def test_rotation_far_out(dim, dims, run):
    """Queries at far positions, some of whose pairs are rotated, ahead of
    their norm."""
    n, rot = 6000, {"base": 50.0, "dims": dims, "scaling": YARN}
    cfg = config((mixer(left(1, 1, dim, 8, 9, 0, dims, 50.0)), None))
    m = build(cfg, run, max_seq=n)
    c, dev, p = m.cache, run[0], m.cache.k[0].shape[3]
    pos = torch.tensor([0, 1, 63, 64, 1000, 4095, 4096, 5999])
    g = torch.Generator().manual_seed(2)
    rows = torch.zeros(len(pos), 3, p)
    rows[..., :dim] = torch.randn(len(pos), 3, dim, generator=g)
    rows = rows.to(element(run))
    slot = c.alloc(n)
    c.extend([slot], [n])
    st = hops.StepMeta(nd=len(pos), pos=pos.to(dev, torch.int32),
                       slot=torch.full((len(pos),), slot, dtype=torch.int32,
                                       device=dev), table=c.table, max_len=n)
    got = hops.qknorm_kv(rows.flatten(1).to(dev), c.k[0], c.v[0], st, 1, 1, dim,
                         1e-3, 0.0, 1, m.rot[0])[:, 0].cpu().double()
    want = oracle.rms(oracle.rotate(rows[:, 0, :dim].double(), pos, rot), 1e-3)
    tol = 2e-5 if run[1] == "fp32" else 0.02
    assert float((got[:, :dim] - want).abs().max()) < tol
    assert not got[:, dim:].any()
    page = c.table[slot].cpu()[pos // 64].long()
    keys = c.k[0].cpu()[page, 0, pos % 64].double()
    want = oracle.rms(oracle.rotate(rows[:, 1, :dim].double(), pos, rot), 1e-3)
    assert float((keys[:, :dim] - want).abs().max()) < tol
    assert torch.equal(c.v[0].cpu()[page, 0, pos % 64], rows[:, 2])


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("width,ns", [(64, 1), (150, 2), (3072, 4), (1026, 3),
                                      (5000, 4), (8192, 2), (8192, 4),
                                      (4096, 7), (128, 16)])
def test_streams(width, ns, run):
    """A sublayer's output (of one row per token, or of several and a gated
    one) joins streams of unlike size."""
    dev, wp, n, eps = run[0], -(-width // 64) * 64, 5, 1e-3
    g = torch.Generator().manual_seed(width + ns)

    def r(*shape):
        t = torch.randn(*shape, width, generator=g)
        return torch.nn.functional.pad(t, (0, wp - width))
    x = r(n, ns) * torch.logspace(-1, 1, ns).view(1, ns, 1)
    w = r() * 0.3 + (torch.arange(wp) < width)
    mix, put, read = (torch.randn(*s, generator=g)
                      for s in ((ns, ns), (ns,), (ns,)))
    hc = torch.cat([mix.flatten(), put]).to(dev)
    tol = 2e-5 if run[1] == "fp32" else 0.03

    def check(got, want):
        assert float((got.cpu()[..., :width].double() - want).abs().max()) \
            < tol * (1 + float(want.abs().max()))
        assert not got[..., width:].any()

    def reads(xs):
        u = torch.einsum("s,nsw->nw", read.double(), xs[..., :width].double())
        return oracle.rms(u, eps) * w[:width].double()

    for top in (0, 1, 3, 9):
        y = r(n * max(1, top)).to(element(run))
        extra, z = None, torch.randn(n, 4, generator=g)
        total = y.double().view(n, max(1, top), wp).sum(1)
        if top % 2:
            extra = r(n).to(element(run))
            total = total + extra.double() * torch.sigmoid(z[:, 2:3]).double()
            extra = (extra.to(dev), z.to(dev)[:, 2:3])
        want = torch.einsum("st,nsw->ntw", mix.double(), x.double()) + \
            put.double().view(1, ns, 1) * total.unsqueeze(1)
        got = x.to(dev).clone()
        h = hops.streams_join(got, y.to(dev), hc, read.to(dev), w.to(dev),
                              width, eps, top, extra)
        err = (got.cpu().double() - want)[..., :width].abs().max()
        assert float(err) < 1e-5 * (1 + float(want.abs().max()))
        check(h, reads(want))
        again = x.to(dev).clone()
        assert hops.streams_join(again, y.to(dev), hc, None, None, width, eps,
                                 top, extra) is None
        assert torch.equal(again, got)
    rows = torch.tensor([3, 0, 3], dtype=torch.int32)
    for at in (None, rows):
        got = hops.streams_norm(x.to(dev), None if at is None else at.to(dev),
                                w.to(dev), width, eps, element(run))
        s = x[..., :width].double().sum(1)
        check(got, (oracle.rms(s, eps) * w[:width].double())[
            slice(None) if at is None else at.long()])
    emb = r(11).to(element(run))
    tok = torch.tensor([10, 0, 3])
    xs, h = hops.streams_start(tok.to(dev), emb.to(dev), 5.5, read.to(dev),
                               w.to(dev), width, eps)
    want = (emb[tok].float() * 5.5).unsqueeze(1).expand(-1, ns, -1)
    assert torch.equal(xs.cpu(), want)
    # (the factors may cancel; what is left then is rounding)
    if abs(float(read.sum())) > 0.3:
        check(h, reads(want))


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("n", [1, 7, 90])
@pytest.mark.parametrize("experts,top", [(6, 2), (19, 1), (70, 5)])
def test_weights_on_the_experts_inputs(experts, top, n, run):
    """Small and large weights against tight limits: weighting the output
    instead, or summing the weights to one, would show."""
    dev, el, (W, F) = run[0], element(run), (64, 128)
    g = torch.Generator().manual_seed(n)
    x = torch.randn(n, W, generator=g).to(el)
    z = torch.randn(n, experts + 1, generator=g) * 3
    gate, up = (torch.randn(experts, F, W, generator=g).to(el) * 0.3
                for _ in "gu")
    down = (torch.randn(experts, W, F, generator=g) * 0.1).to(el)
    both = torch.stack([gate.view(experts, -1, 16, W),
                        up.view(experts, -1, 16, W)], dim=2).reshape(
                            experts, 2 * F, W)
    how = Choice(top, sigmoid=True, weigh_input=True,
                 glu=Glu(1.702, 0.8, 1.0, 0.0))
    y, wt, ident = hops.moe(x.to(dev), z.to(dev)[:, :experts], both.to(dev),
                            down.to(dev), how)
    at, s = oracle.choose(z[:, :experts].double(), top)
    assert ident is None
    assert float((wt.cpu().double() - s).abs().max()) < 1e-6
    for t in range(n):
        for k in range(top):
            e = int(at[t, k])
            want = oracle.expert(s[t, k] * x[t].double(), {
                "gate": gate[e].double(), "up": up[e].double(),
                "down": down[e].double()}, 0.8)
            assert float(errors(y[t * top + k][None], want[None])) < \
                (1e-5 if run[1] == "fp32" else 0.02)


# -------------------------------------------- keys and tokens that stand out

CUTS = {"whole": [330], "decode-tail": [185, 1], "pairs": [250, 2],
        "odd": [63, 2, 1, 64, 65]}


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("how", sorted(CUTS))
@pytest.mark.parametrize("sizes", [
    (6, 2, 64, 40, 100, 7, 64), (24, 8, 128, 128, 64, 64, 32),
    (11, 1, 48, 64, 33, 0, 16), (2, 1, 160, 200, 1, 90, 96),
    (3, 3, 20, 20, 500, 2, 20)], ids=str)
def test_one_key_stands_out(sizes, how, run):
    """Every query looks for one key: the first ones, the last kept and the
    next, the window's edges from both sides, page borders, itself, its
    neighbours, also the next one, which it must not see."""
    dev, dtype = run
    el = element(run)
    (H, G, d, dv, size, keep, dims), n, eps = sizes, 330, 1e-5
    a = left(H, G, d, dv, size, keep, dims, 30.0, 24.0 / d)
    m = build(config((mixer(a), None)), run, max_seq=n)
    m.cache.alloc(70)                     # page 1 and 2 belong to another
    c, slot, p = m.cache, m.cache.alloc(0), m.cache.k[0].shape[3]
    g = torch.Generator().manual_seed(5)
    pos = torch.arange(n)
    v = torch.randn(n, G, dv, generator=g).to(el)
    gate = torch.randn(n, H, dv, generator=g).to(el)
    k = torch.randn(n, G, d, generator=g).to(el)
    turned = oracle.rotate(k.double(), pos, a["rot"])
    q = torch.zeros(n, H, d, dtype=torch.float64)
    for h in range(H):
        aim = []
        for i in range(n):
            t = [0, keep - 1, keep, i - size + 1, i - size, i, i - 1, i + 1,
                 i // 64 * 64, i // 64 * 64 - 1, 64, 63]
            t = [j for j in t if 0 <= j < n]
            aim.append(t[(i * 7 + h * 5) % len(t)])
        # turned back from the query's own position
        q[:, h] = oracle.rotate(turned[aim, h // (H // G)], -pos, a["rot"])
    q = oracle.rms(q, eps).to(el)
    want = oracle.attend(
        oracle.rms(oracle.rotate(q.double(), pos, a["rot"]), eps),
        oracle.rms(turned, eps), v.double(), a["scale"],
        oracle.visible(n, n, size, keep)) * torch.sigmoid(gate.double())

    def lay(t):
        return torch.nn.functional.pad(t, (0, p - t.shape[2])).flatten(1)
    rows = torch.cat([lay(q), lay(k), lay(v), lay(gate),
                      torch.zeros(n, 64, dtype=el)], dim=1)
    got, end = [], (2 * H + 2 * G) * p
    for at, ln in portions(n, CUTS[how]):
        c.extend([slot], [ln])
        st = meta_for(c, slot, at, ln, dev)
        part = rows[at:at + ln].to(dev).contiguous()
        pq = hops.qknorm_kv(part, c.k[0], c.v[0], st, H, G, d, eps, 0.0, 1,
                            m.rot[0])
        out = torch.full((ln, H * p + 64), 9.0, dtype=el, device=dev)
        hops.paged_attn(pq, c.k[0], c.v[0], st, a["scale"], None,
                        part[:, end - H * p:end], Keys(size, keep),
                        out[:, :H * p], 0.5)
        assert (out[:, H * p:] == 9.0).all()
        got.append(out[:, :H * p].view(ln, H, p))
    got = torch.cat(got).cpu().double()
    assert not got[..., dv:].any()
    err = (got[..., :dv] - 0.5 * want).abs().amax(-1)
    assert float(err.max()) < (1e-4 if dtype == "fp32" else 0.06)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("how", sorted(CUTS))
@pytest.mark.parametrize("H,dk,dv", [(4, 64, 64), (6, 128, 256), (2, 192, 64)])
def test_one_token_stands_out_in_the_memory(H, dk, dv, how, run):
    """Decays from nothing kept to everything kept; a few loud tokens at chunk
    and page borders, which later queries find. What the state holds is exact
    to rounding of the inputs and the result."""
    dev, n, el = run[0], 330, element(run)
    decay = ([1.0, 0.999, 0.9, 0.0, 0.3, 0.99] * 2)[:H]
    g = torch.Generator().manual_seed(H)
    rows = torch.randn(n, 2 * H * (dk + dv) + 64, generator=g)
    loud = [0, 1, 62, 63, 64, 127, 128, 200]
    at = 2 * H * dk
    rows[loud, at:at + H * dv] *= 30
    rows[:, :at] *= 0.3
    for t in range(n):                     # look for one of them
        rows[t, :H * dk] += 3 * rows[loud[t % len(loud)], H * dk:at]
    rows = rows.to(el)
    count = at + H * dv
    acted = oracle.silu(rows[:, :count].double())
    if run[1] == "bf16":
        acted = acted.to(el).double()
    q, k, v = (t.view(n, H, -1) for t in
               acted.split([H * dk, H * dk, H * dv], 1))
    o = oracle.decaying_memory(q, k, v, decay).reshape(n, -1)
    norm = torch.rand(H * dv, generator=g) + 0.5
    gates = rows[:, count:count + H * dv].double()
    want = oracle.rms(o, 1e-5) * norm.double() * torch.sigmoid(gates)
    cfg = config((mixer(b=right(H, dk, dv, decay)), None))
    m = build(cfg, run, max_seq=n)
    c, slot = m.cache, m.cache.alloc(0)
    c.S[0].fill_(7.0)                      # of no matter to a new sequence
    two = m.layers[0].decay
    got = []
    for p0, ln in portions(n, CUTS[how]):
        c.extend([slot], [ln])
        st = meta_for(c, slot, p0, ln, dev)
        part = rows[p0:p0 + ln].to(dev).contiguous()
        hops.silu_cols(part, 0, count)
        out = torch.full((ln, H * dv + 64), 9.0, dtype=el, device=dev)
        hops.lightning(part, c.S[0], two, norm.to(dev), st, dv, 1e-5,
                       out[:, :H * dv])
        assert (out[:, H * dv:] == 9.0).all()
        got.append(out[:, :H * dv])
    e = errors(torch.cat(got), want)
    assert float(e.max()) < (2e-5 if run[1] == "fp32" else 0.004)
    others = [s for s in range(c.slots) if s != slot]
    assert (c.S[0][others] == 7.0).all()


# ----------------------------------------------- cuts, batches, pages, slots

@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("sizes", [[1], [2], [3], [63, 2], [64], [100, 1],
                                   [16, 17], [130, 1, 7]], ids=str)
def test_cuts_do_not_matter(sizes, run):
    m = build(FULL, run)
    ids = tokens(140, seed=1)
    want, _ = oracle.forward(FULL, weights_of(FULL), ids)
    slot = m.cache.alloc(0)
    close(feed(m, slot, ids, sizes), want, run)


@pytest.mark.parametrize("run", RUNS)
def test_unequal_batch_against_each_alone(run):
    m = build(FULL, run)
    seqs = {s: tokens(n, seed=s) for s, n in ((1, 150), (2, 3), (3, 70),
                                              (4, 97))}
    want = {s: oracle.forward(FULL, weights_of(FULL), ids)[0]
            for s, ids in seqs.items()}
    # portions of some beside single tokens of others; one pauses
    steps = [{1: 64, 2: 1, 3: 2}, {1: 5, 3: 63, 4: 30}, {1: 1, 3: 1, 4: 2},
             {1: 60, 2: 1, 4: 64}, {1: 1, 2: 1, 3: 1, 4: 1}, {3: 2}, {1: 18},
             {1: 1, 3: 1}]
    slots = {s: m.cache.alloc(0) for s in seqs}
    at = {s: 0 for s in seqs}
    got = {s: [] for s in seqs}
    for st in steps:
        out = m.forward_step([(slots[s], seqs[s][at[s]:at[s] + n],
                               list(range(n))) for s, n in st.items()]).cpu()
        for (s, n), part in zip(st.items(), out.split(list(st.values()))):
            got[s].append(part)
            at[s] += n
    assert at == {s: len(v) for s, v in seqs.items()}
    for s in seqs:
        close(torch.cat(got[s]), want[s], run)
    close(whole(m, seqs[3]), want[3], run)     # in the slot that is left


@pytest.mark.parametrize("run", RUNS)
def test_pages_and_slots_are_used_again(run):
    """A pool that only fits if everything is given back, in an order that
    scatters the pages of later sequences."""
    m = build(FULL, run, slots=3, pool=64 * 7)
    first = {}
    for rnd in range(3):
        s1, s2 = m.cache.alloc(0), m.cache.alloc(0)
        a, b = tokens(150, seed=10), tokens(140, seed=11)
        ga, gb = [], []
        for i in range(0, 150, 30):           # interleave the page demand
            ga.append(m.forward_step([(s1, a[i:i + 30], [0, 29])]))
            if i < 140:
                part = b[i:i + 30]
                gb.append(m.forward_step([(s2, part, [len(part) - 1])]))
        for key, out in (("a", ga), ("b", gb)):
            out = torch.cat(out).cpu()
            close(out, first.setdefault(key, out), run, exact=1e-4)
        m.cache.free(s2 if rnd else s1)
        s3 = m.cache.alloc(0)
        c = tokens(130, seed=12)
        close(feed(m, s3, c, [100, 1])[[0, 129]],
              oracle.forward(FULL, weights_of(FULL), c)[0][[0, 129]], run)
        m.cache.free(s3)
        m.cache.free(s1 if rnd else s2)
    assert len(m.cache._free_pages) == 7 and m.cache.n_free == 1


@pytest.mark.parametrize("run", EXACT)
def test_long_decode(run):
    """Token by token from the first one on, over several pages, chunks and
    windows."""
    cfg = config((mixer(left(size=70, keep=3)), moe()),
                 (mixer(left(2, 1, size=50, keep=66)), None), loop=(0, 1, 2))
    m = build(cfg, run)
    ids = tokens(270, cfg, seed=4)
    slot = m.cache.alloc(0)
    close(feed(m, slot, ids, [1]), oracle.forward(cfg, weights_of(cfg), ids)[0],
          run)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("heads,kv,dim,size,keep", [
    (24, 8, 32, 900, 100), (4, 1, 72, 130, 300), (2, 2, 16, 1999, 0)])
def test_long_windows(heads, kv, dim, size, keep, run):
    """Decoding splits the keys of a window, and prompts take many tiles."""
    cfg = config((mixer(left(heads, kv, dim, dim, size, keep, 16, scale=0.5)),
                  None))
    W = weights_of(cfg)
    m = build(cfg, run, W=W, max_seq=2200)
    ids = tokens(2100 if run[0] != "cpu" else 720, cfg, seed=7)
    slot, at, got, places = m.cache.alloc(0), 0, [], []
    for n in [699, 1, 1, 1299, 1, 1, 17, 2, 1]:
        part = ids[at:at + n]
        if not part:
            break
        where = sorted({0, len(part) // 2, len(part) - 1})
        got.append(m.forward_step([(slot, part, where)]).cpu())
        places += [at + i for i in where]
        at += len(part)
    close(torch.cat(got),
          oracle.forward(cfg, W, ids[:at], torch.float32)[0][places], run)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("heads,kv", [(4, 2), (16, 8)])
def test_many_rows_decode_at_once(heads, kv, run):
    """Enough rows that no row's keys are split."""
    n = 290 if run[0] != "cpu" else 12
    cfg = config((mixer(left(heads, kv, 16, 16)), moe()), ONE)
    m = build(cfg, run, slots=n, max_seq=128)
    seqs = [tokens(k, cfg, seed=k) for k in (71, 3, 40)]
    slots = [m.cache.alloc(0) for _ in range(n)]
    m.forward_step([(s, seqs[i % 3][:-1], []) for i, s in enumerate(slots)])
    got = m.forward_step([(s, seqs[i % 3][-1:], [0])
                          for i, s in enumerate(slots)])
    want = [oracle.forward(cfg, weights_of(cfg), q)[0][-1] for q in seqs]
    close(got, torch.stack([want[i % 3] for i in range(n)]), run)


# ------------------------------------------------- configuration and weights

def test_config_reader():
    W = weights_of(FULL)
    spec = read_zinavik(FULL)
    assert spec.params == sum(v.numel() for v in W.values())
    assert [ly.mixer.left.window for ly in spec.layers] == \
        [37, 100, 12, 100, 12, 100, 12, 1]
    assert [spec.number(spec.owner(i)) for i in range(8)] == \
        oracle.order_of(FULL)
    m = HybridModel(spec, dtype="fp32", random_init=False, kv_tokens=256)
    assert m.tensor_shapes() == {k: tuple(v.shape) for k, v in W.items()}
    assert ops_build.libs_of(spec) == ["hip", "hybrid"]

    def broken(change):
        c = json.loads(json.dumps(FULL))
        change(c)
        with pytest.raises((ValueError, KeyError)):
            read_zinavik(c)

    def mx(c, side="left", i=0):
        return c["layers"][i]["mixer"][side]

    broken(lambda c: c.pop("streams"))
    broken(lambda c: c.update(streams=0))
    broken(lambda c: c.update(streams=17))
    broken(lambda c: c.update(window=3))
    broken(lambda c: c["embedding"].pop("scale"))
    broken(lambda c: c["norm"].update(groups=3))
    broken(lambda c: c["loop"].update(stop=1))
    broken(lambda c: c["loop"].update(stop=5))
    broken(lambda c: c["loop"].update(times=0))
    broken(lambda c: c["layers"][0].update(type="left"))
    broken(lambda c: c["layers"][0]["mixer"].pop("left_scale"))
    broken(lambda c: mx(c).update(kv_heads=3))
    broken(lambda c: mx(c).update(softcap=3))
    broken(lambda c: mx(c)["rot"].update(dims=15))
    broken(lambda c: mx(c)["rot"].update(dims=34))
    broken(lambda c: mx(c)["rot"]["scaling"].pop("slow"))
    broken(lambda c: mx(c)["mask"].update(size=0))
    broken(lambda c: mx(c)["mask"].update(keep_first=-1))
    broken(lambda c: mx(c, "right").update(decay=[0.5, 0.5]))
    broken(lambda c: mx(c, "right").update(decay=[0.5, 0.5, 1.5]))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="dense"))
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=4))
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(groups=7))
    broken(lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"))


def test_specs_that_make_no_sense():
    spec = read_zinavik(FULL)
    for wrong in (dict(streams=0), dict(pre_norms=True), dict(positions=64),
                  dict(plain_norms=False), dict(post_alpha=1.0),
                  dict(depth_average=True), dict(embed_norm=True),
                  dict(layers=(spec.layers[0], replace(spec.layers[1],
                                                       number=0)))):
        with pytest.raises(ValueError):
            replace(spec, **wrong)
    assert [ly.weights_of for ly in looped([spec.layers[0]] * 2, 0, 2, 2)] == \
        [None, None, 0, 1]


def test_every_pass_has_a_cache_of_its_own():
    m = HybridModel(read_zinavik(FULL), dtype="fp32", random_init=False,
                    kv_tokens=256)
    kv = [t.data_ptr() for t in m.cache.k + m.cache.v + m.cache.S]
    assert len(set(kv)) == 3 * 8
    per = []
    for ly, p in zip(m.spec.layers, (64, 128, 128, 128, 128, 128, 128, 64)):
        b = ly.mixer.right
        pad = [-(-x // 64) * 64 for x in (b.dim, b.vdim)]
        per.append(4 * (2 * 5 * ly.mixer.left.kv_heads * 64 * p +
                        64 * b.heads * pad[0] * pad[1]))
    assert m.cache.bytes() == sum(per)


@pytest.mark.parametrize("run", RUNS)
def test_lightning_attention_as_a_layer_of_its_own(run):
    b = right(2, 24, 40, (0.6, 0.99))
    cfg = config((mixer(left(), b), None))
    W = {k.replace("mix.right.", "mix."): v
         for k, v in weights_of(cfg).items() if "mix.left" not in k}
    spec = HybridSpec("lightning-alone", vocab=130, hidden=96, norm_eps=1e-5,
                      layers=(LayerSpec(LightningMixer(2, 24, 40, (0.6, 0.99)),
                                        DenseFF(64, 2.0)),), streams=3,
                      embed_scale=7.0, plain_norms=True, max_seq_len=256)
    g = torch.Generator().manual_seed(3)
    extra = {"gate": (64, 96), "up": (64, 96), "down": (96, 64)}
    W |= {"l0.mlp." + k: torch.randn(s, generator=g) * 0.1
          for k, s in extra.items()}
    W |= {"l0.norm2": W["l0.norm1"] * 0.8} | {
        f"l0.hc2.{k}": W[f"l0.hc1.{k}"] * 0.9 for k in ("in", "out", "mix")}
    W = {k: v.to(torch.bfloat16) for k, v in W.items()}
    m = HybridModel(spec, device=run[0], dtype=run[1], kv_slots=2,
                    random_init=False)
    assert m.tensor_shapes() == {k: tuple(v.shape) for k, v in W.items()}
    assert spec.params == sum(v.numel() for v in W.values())
    m._assemble(lambda name: W[name].to(run[0]))
    ids = tokens(100, cfg)
    got = feed(m, m.cache.alloc(0), ids, [80, 3, 1])
    D = {k: v.double() for k, v in W.items()}
    xs = torch.stack([D["embed"][ids] * 7.0] * 3)
    wm, we = oracle._under(D, "l0.mix."), oracle._under(D, "l0.mlp.")
    xs = oracle.sublayer(xs, oracle._under(D, "l0.hc1."), D["l0.norm1"], 1e-5,
                         lambda h: oracle.lightning(h, wm, b, 1e-5)
                         @ wm["o"].T)
    xs = oracle.sublayer(xs, oracle._under(D, "l0.hc2."), D["l0.norm2"], 1e-5,
                         lambda h: oracle.expert(h, we, 2.0))
    close(got, oracle.rms(xs.sum(0), 1e-5) * D["final.norm"] @ D["embed"].T,
          run)


@pytest.fixture
def checkpoint(tmp_path):
    from safetensors.torch import save_file
    save_file(weights_of(FULL, 3), str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(FULL))
    return tmp_path


def test_checkpoint_describes_itself(checkpoint):
    spec = resolve_spec("llama3.2:1b", str(checkpoint))
    assert (spec.family, spec.name) == ("zinavik", "zinavik:custom")
    m = HybridModel(spec, dtype="fp32", random_init=False, kv_tokens=256)
    assert m.load_safetensors(str(checkpoint)) == len(weights_of(FULL))
    from safetensors.torch import save_file
    W = weights_of(FULL, 3)
    del W["l3.hc2.mix"]
    save_file(W, str(checkpoint / "model.safetensors"))
    with pytest.raises(KeyError, match="l3.hc2.mix"):
        m.load_safetensors(str(checkpoint))


# --------------------------------------------------- engine and its schedule

def engine_for(checkpoint, run, **kw):
    kw = {"max_seq_len": 256, "max_batch_size": 4, "autotune": False} | kw
    return InferenceEngine(EngineConfig(
        weights_path=str(checkpoint), device=run[0], dtype=run[1], **kw))


def greedy(ids, steps, seed=3):
    """Greedy continuation by the plain implementation, and how far the
    winner stood above the second at each step."""
    W, ids, gaps = weights_of(FULL, seed), list(ids), []
    for _ in range(steps):
        z = oracle.forward(FULL, W, ids)[0][-1]
        top = torch.topk(z, 2)
        gaps.append(float(top.values[0] - top.values[1]))
        ids.append(int(top.indices[0]))
    return ids[-steps:], gaps


GREEDY = {"temperature": 0.0, "num_predict": 6}
PROMPTS = ["2 + 3 = ", "q", "A prompt that is long enough to take more than "
           "one page of the cache and several portions ...", "?"]


@pytest.mark.parametrize("run", EXACT)
@pytest.mark.parametrize("chunk", [8192, 5])
def test_greedy_generation(checkpoint, run, chunk):
    """Through generate, generate_batch and the continuous batcher, with whole
    prompts and with portions of five tokens beside decoding rows."""
    from gridllm_amd.engine.batcher import Batcher
    eng = engine_for(checkpoint, run, prefill_chunk=chunk)
    eng.tokenizer = Bytes(FULL["vocab"])
    want, gaps = zip(*(greedy(eng.tokenizer.encode(p), 6) for p in PROMPTS))
    assert min(min(g) for g in gaps) > 1e-3        # no close call in the test
    free = eng.model.cache.n_free
    assert [eng.generate(p, GREEDY).token_ids for p in PROMPTS] == list(want)
    out = eng.generate_batch([(p, GREEDY) for p in PROMPTS])
    assert [r.token_ids for r in out] == list(want)
    b = Batcher(eng)
    try:
        futs = [b.submit_generate(p, GREEDY) for p in PROMPTS * 3]
        assert [f.result(60).token_ids for f in futs] == list(want) * 3
        deadline = time.time() + 10
        while eng.model.cache.n_free != free and time.time() < deadline:
            time.sleep(0.02)
    finally:
        b.shutdown()
    assert eng.model.cache.n_free == free
    assert len(eng.embed(["abc", "defg"])[1]) == FULL["width"]


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("name", ["tiny-zinavik", "tiny-zinavik:latest"])
def test_registered_model_serves(name, run):
    eng = InferenceEngine(EngineConfig(model=name, device=run[0], dtype=run[1],
                                       max_batch_size=2, max_seq_len=128))
    r = eng.generate("hello", {"temperature": 0.7, "seed": 5,
                               "num_predict": 6})
    assert r.eval_count == 6
    assert "tiny-zinavik" in eng.model_names()
    info = eng.spec.model_info()
    assert info["general.architecture"] == "zinavik"
    assert info["zinavik.attention.sliding_window"] == 48
    assert info["zinavik.block_count"] == 4
    assert get_spec("zinavik:4b").params > 4e9


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_long_decode_by_captured_graphs(checkpoint, dtype):
    """Decode-only steps replay captured graphs, between eager mixed steps and
    synchronizations; every step against the eager model, 150 tokens long and
    over page, window and chunk borders."""
    run = ("cuda:0", dtype)
    eng = engine_for(checkpoint, run)
    assert eng._graph_ok() and eng._graphs
    W = weights_of(FULL, 3)
    ref = build(FULL, run, W=W)
    ids = {i: tokens(190, seed=20 + i) for i in range(3)}
    a = {i: eng.open_sequence() for i in ids}
    b = {i: ref.cache.alloc(0) for i in ids}
    at = {0: 40, 1: 2, 2: 33}
    got, want = [], []
    eng.run_step([(a[i], ids[i][:n], []) for i, n in at.items()])
    ref.forward_step([(b[i], ids[i][:n], []) for i, n in at.items()])
    for step in range(150):
        live = [i for i in ids if not (i == 1 and step % 3 == 0)]
        n = {i: 2 if step % 31 == 30 and i == 2 else 1 for i in live}
        ent = [(i, ids[i][at[i]:at[i] + n[i]], [0]) for i in live
               if at[i] + n[i] <= 190]
        got.append(eng.run_step([(a[i], t, w) for i, t, w in ent]).clone())
        want.append(ref.forward_step([(b[i], t, w) for i, t, w in ent]))
        for i, t, _ in ent:
            at[i] += len(t)
        if step % 10 == 0:
            torch.cuda.synchronize()
    close(torch.cat(got), torch.cat(want).cpu(), run, exact=1e-4)
    close(eng.run_step([(a[0], [7], [0])]),
          oracle.forward(FULL, W, ids[0][:at[0]] + [7])[0][-1:], run)


@pytest.mark.parametrize("run", RUNS)
def test_trace_replay(checkpoint, tmp_path, run):
    from gridllm_amd import trace
    a, b = tokens(80, seed=1), tokens(3, seed=2)
    steps = [{"step": 0, "entries": [
                 {"id": "a", "tokens": a[:70], "want": [0, 69]},
                 {"id": "b", "tokens": b[:1], "want": [0]}], "end": []},
             {"step": 1, "entries": [
                 {"id": "b", "tokens": b[1:], "want": []}], "end": ["b"]},
             {"step": 2, "entries": [
                 {"id": "a", "tokens": a[70:71], "want": [0]}], "end": []},
             {"step": 3, "entries": [
                 {"id": "c", "tokens": b, "want": [2]},
                 {"id": "a", "tokens": a[71:], "want": [8]}],
              "end": ["a", "c"]}]
    W = weights_of(FULL, 3)
    la, lb = (oracle.forward(FULL, W, t)[0] for t in (a, b))
    want = {0: torch.stack([la[0], la[69], lb[0]]), 2: la[70:71],
            3: torch.stack([lb[2], la[79]])}
    out = tmp_path / "out"
    out.mkdir()
    eng = trace.make_engine(str(checkpoint),
                            {"fp32": "float32", "bf16": "bfloat16"}[run[1]],
                            256, run[0])
    acks = io.StringIO()
    trace.replay(eng, io.StringIO("".join(json.dumps(s) + "\n"
                                          for s in steps)), str(out), acks)
    assert acks.getvalue() == "".join(f"done {i}\n" for i in range(4))
    assert len(eng.model.cache._free_pages) == eng.model.cache.pages == 4
    assert sorted(os.listdir(out)) == [f"{k}.f32" for k in sorted(want)]
    for k, w in want.items():
        got = np.fromfile(os.path.join(out, f"{k}.f32"), dtype="<f4")
        close(torch.from_numpy(got).view(w.shape), w, run)
