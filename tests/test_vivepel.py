"""Vivepel against the plain implementation in vivepel_oracle: on the CPU in
f32, on the GPU in f32 and bf16."""

import io
import json
import math
import os
import sys
import time

import numpy as np
import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import vivepel_oracle as oracle  # noqa: E402
from hybrid_helpers import (EXACT, RUNS, Bytes, close, errors,  # noqa: E402
                            feed, meta_for, one_thread, portions,  # noqa: F401
                            whole)

from gridllm_amd.config import EngineConfig  # noqa: E402
from gridllm_amd.engine import InferenceEngine  # noqa: E402
from gridllm_amd.models.hybrid import HybridModel, _pair_order  # noqa: E402
from gridllm_amd.models.registry import (get_spec, read_vivepel,  # noqa: E402
                                         resolve_spec)
from gridllm_amd.ops import build as ops_build  # noqa: E402
from gridllm_amd.ops import hybrid as hops  # noqa: E402


def attn(heads=4, kv_heads=2, dim=32, chunk=40, rot=16, base=3000.0,
         scale=0.2, cap=12.0):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim,
            "scale": scale, "softcap": cap, "mask": {"size": chunk},
            "rot": {"base": base, "dims": rot}}


def dense(ff=96):
    return {"kind": "dense", "ff": ff}


def config(*layers, vocab=130, width=96, eps=1e-5, groups=3):
    return {"architecture": "Vivepel", "vocab": vocab, "width": width,
            "norm": {"eps": eps, "groups": groups},
            "layers": [{"type": "attention", "mixer": m, "mlp": f}
                       for m, f in layers]}


# layers of unlike sizes, with and without a feed-forward, that need padding
FULL = config((attn(), dense()),
              (attn(3, 1, 40, 100, 24, 50.0, 0.3, 5.0), None),
              (attn(5, 5, 72, 64, 72, 1e4, 0.1, 50.0), dense(200)),
              (attn(9, 3, 20, 7, 6), dense(40)),
              (attn(2, 2, 16, 1000, 2, cap=8.0), dense()))


def weights_of(cfg, seed=0):
    return oracle.random_weights(cfg, seed)


def build(cfg, run, seed=0, slots=5, pool=0, W=None, max_seq=512):
    dev, dtype = run
    W = W or weights_of(cfg, seed)
    m = HybridModel(read_vivepel(cfg), device=dev, dtype=dtype,
                    kv_slots=slots, kv_tokens=pool, max_seq=max_seq,
                    random_init=False)
    m._assemble(lambda name: W[name].to(dev))
    return m


def tokens(n, cfg=FULL, seed=0):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


# ------------------------------------------------------------ each mechanism

ALONE = {
    "attention": config((attn(), None)),
    "one-head": config((attn(1, 1, 64), None)),
    "one-value-head": config((attn(7, 1, 24, rot=8), None)),
    "no-groups-of-heads": config((attn(6, 6, 16), None)),
    "heads-over-waves": config((attn(20, 4, 16, rot=12), None)),
    "most-tiled-heads": config((attn(32, 8, 24, rot=10), None)),
    "more-heads-than-tiled": config((attn(33, 3, 16), None)),
    "most-heads": config((attn(64, 8, 16), None)),
    "more-heads-than-decoded": config((attn(66, 2, 8, rot=8), None)),
    "many-value-heads": config((attn(16, 16, 16), None)),
    "seventeen-value-heads": config((attn(17, 17, 16), None)),
    "padded-head": config((attn(4, 2, 72, rot=36), None)),
    "wide-head": config((attn(4, 2, 160, rot=64, scale=0.05), None)),
    "wide-head-many-heads": config((attn(18, 2, 130, rot=2, scale=0.05),
                                    None)),
    "no-rotation": config((attn(rot=0), None)),
    "full-rotation": config((attn(rot=32, base=3.0), None)),
    "one-pair": config((attn(rot=2), None)),
    "chunk-of-one": config((attn(chunk=1), None)),
    "chunk-of-five": config((attn(chunk=5), None)),
    "chunk-of-a-page": config((attn(chunk=64), None)),
    "chunk-beyond-all": config((attn(chunk=5000), None)),
    "tight-cap": config((attn(cap=0.5, scale=1.0), None)),
    "loose-cap": config((attn(cap=100.0, scale=1.5), None)),
    "no-tiles-cap": config((attn(cap=300.0, scale=2.0), None)),
    "dense": config((attn(1, 1, 16), dense(200))),
    "dense-wide": config((attn(1, 1, 16), dense(5000)), width=64, groups=2),
    "one-norm-group": config((attn(), dense()), groups=1, width=200),
    "groups-of-two": config((attn(), dense()), groups=48, eps=0.1),
    "groups-of-one": config((attn(), dense()), groups=96, eps=0.3),
    "odd-groups": config((attn(), dense()), groups=3, width=75),
    "coarse-eps": config((attn(), dense()), eps=0.05),
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
    for a, b in zip(trail, layers):
        close(a, b, run)
    close(got, want, run)


def element(run):
    return torch.float32 if run[1] == "fp32" else torch.bfloat16


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("width,groups", [
    (64, 1), (192, 3), (150, 5), (75, 3), (8192, 16), (3072, 2), (1026, 57)])
def test_group_norms(width, groups, run):
    """Norm of the sum and of a sublayer's output, groups of unlike size of
    their values, at picked rows and at all."""
    dev, wp, n = run[0], -(-width // 64) * 64, 5
    g = torch.Generator().manual_seed(width)
    loud = torch.logspace(-2, 2, groups).repeat_interleave(width // groups)

    def pad(t):
        return torch.nn.functional.pad(t, (0, wp - width))
    x = pad(torch.randn(n, width, generator=g) * loud)
    y = pad(torch.randn(n, width, generator=g) * loud.flip(0)).to(element(run))
    wy, w = (pad(1 + 0.3 * torch.randn(width, generator=g)) for _ in "ab")
    how = (groups, width, 1e-3)
    rows = torch.tensor([3, 0, 3], dtype=torch.int32)

    def norm(t, v):
        return oracle.group_norm(t[:, :width].double(), v[:width].double(),
                                 groups, 1e-3)
    tol = 1e-5 if run[1] == "fp32" else 0.02
    got = hops.group_norm(x.to(dev), rows.to(dev), w.to(dev), *how,
                          element(run)).cpu()
    want = norm(x[[3, 0, 3]], w)
    assert float((got[:, :width] - want).abs().max()) < tol * 5
    assert not got[:, width:].any()
    x2 = x.to(dev).clone()
    h = hops.join_norm(x2, y.to(dev), wy.to(dev), w.to(dev), *how).cpu()
    want = x[:, :width].double() + norm(y, wy)
    assert float((x2.cpu()[:, :width] - want).abs().max()) < 1e-4
    assert float((h[:, :width] - norm(want, w)).abs().max()) < tol * 5
    assert not h[:, width:].any() and not x2[:, width:].any()
    x3 = x.to(dev).clone()
    assert hops.join_norm(x3, y.to(dev), wy.to(dev), None, *how) is None
    assert torch.equal(x2, x3)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("ff", [40, 64, 4096, 5000, 16384, 20000])
def test_poly_norm(ff, run):
    fp = -(-ff // 64) * 64
    g = torch.Generator().manual_seed(ff)
    z = torch.nn.functional.pad(torch.randn(7, ff, generator=g) *
                                torch.logspace(-3, 1, 7).view(7, 1),
                                (0, fp - ff)).to(element(run))
    coef = torch.tensor([0.7, -0.4, 0.3, 0.2])
    want = oracle.poly_norm(z[:, :ff].double(), coef.double(), 1e-3)
    got = hops.poly_norm(z.to(run[0]), coef.to(run[0]), ff, 1e-3)[:, :ff]
    assert got.dtype == z.dtype
    assert float(errors(got, want).max()) < \
        (1e-5 if run[1] == "fp32" else 0.005)


# ------------------------------------------------------ keys that stand out

CUTS = {"whole": [330], "decode-tail": [185, 1], "pairs": [250, 2],
        "sixteens": [90, 16, 17], "odd": [63, 2, 1, 64, 65]}


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("how", sorted(CUTS))
@pytest.mark.parametrize("sizes", [
    (4, 2, 64, 100, 64), (24, 8, 128, 96, 40), (20, 4, 48, 33, 16),
    (40, 2, 64, 64, 32), (2, 1, 160, 1000, 96), (32, 16, 64, 200, 0)], ids=str)
def test_one_key_stands_out(sizes, how, run):
    """Every query looks for one key: the first, the neighbours of page and
    chunk borders, itself, the previous one; for some it is the next one, or
    the last of the chunk before, which it must not see. Far positions, so that
    rotations by one position too few would show."""
    dev, dtype = run
    el = element(run)
    (H, G, d, chunk, rot), n, base = sizes, 330, 30.0
    pd = 64 if d <= 64 else 128 if d <= 128 else 256
    cfg = config((attn(H, G, d, chunk, rot, base, 24.0 / d, 30.0), None))
    W = weights_of(cfg, 2)
    m = build(cfg, run, W=W, max_seq=n)
    m.cache.alloc(70)                     # page 1 and 2 belong to another
    cache, w, slot = m.cache, m.layers[0], m.cache.alloc(0)
    g = torch.Generator().manual_seed(5)
    pos, eps = torch.arange(n), cfg["norm"]["eps"]
    qn, kn = (W[f"l0.mix.{c}.norm"].double() for c in "qk")
    bias = torch.cat([W["l0.mix.q.b"], W["l0.mix.k.b"]]).double()
    v = torch.randn(n, G, d, generator=g).double()
    k = oracle.keys_of(v, kn, pos, base, rot, eps)
    border = sorted({b + o for b in [*range(0, n, 64), *range(0, n, chunk)]
                     for o in (-2, -1, 0, 1)} & set(range(n)))
    q = torch.zeros(n, H, d, dtype=torch.float64)
    for h in range(H):
        aim = []
        for p in range(n):
            targets = [t for t in border if p - 2 * chunk <= t <= p + 1]
            targets += [p, max(p - 1, 0), min(p + 1, n - 1),
                        max(p // chunk * chunk - 1, 0), p // chunk * chunk]
            aim.append(targets[(p * 7 + h * 5) % len(targets)])
        # turned back from the query's own position, ahead of norm and weight
        q[:, h] = oracle.rotate_half(k[aim, h * G // H], -pos, base, rot) / qn
    rows = torch.cat([q.flatten(1), v.flatten(1)], 1) - bias
    rows = rows.to(el)
    # what the layer sees after rounding
    cols = rows.double() + bias
    qd, vd = cols.split([H * d, G * d], dim=1)
    vd = vd.view(n, G, d).to(el).double()
    talk = W["l0.mix.talk"].double()
    want = oracle.attend(
        oracle.keys_of(qd.view(n, H, d), qn, pos, base, rot, eps),
        oracle.keys_of(vd, kn, pos, base, rot, eps), vd, talk, 24.0 / d, 30.0,
        chunk)
    order = _pair_order(d, rot)
    laid = torch.zeros(n, H + G, pd, dtype=el)
    laid[..., :d] = rows.view(n, H + G, d)[..., order]
    laid = torch.nn.functional.pad(laid.flatten(1), (0, 64))
    got = []
    for at, ln in portions(n, CUTS[how]):
        cache.extend([slot], [ln])
        st = meta_for(cache, slot, at, ln, dev, chunk=chunk)
        if dtype == "fp32" or at % 3 == 0:     # where nothing is laid out
            st.talk = {}
            st.absorbed = ln
        part = hops.talk_rows(laid[at:at + ln].to(dev).contiguous(),
                              cache.v[0], cache.inv[0], st, w.talk, eps)
        got.append(hops.talk_attn(part, cache.v[0], cache.inv[0], st, w.talk))
    got = torch.cat(got).cpu().double()
    assert not got[..., d:].any()
    err = (got[..., :d] - want[..., order]).abs().amax(-1)
    # (mixing adds up errors of all heads' weights)
    assert float(err.max()) < \
        (2e-4 if dtype == "fp32" else 0.05 + 0.01 * math.sqrt(H))


@pytest.mark.parametrize("run", RUNS)
def test_the_sink_takes_its_share(run):
    """Scores near the lower cap: nearly all weight goes to the sink, whose
    share no mixing brings back."""
    cfg = config((attn(2, 1, 32, 50, 0, scale=0.5, cap=9.0), None))
    W = weights_of(cfg)
    # queries and keys from the biases alone, opposite to each other
    for k in ("l0.mix.q", "l0.mix.k"):
        W[k] = W[k] * 0.0
    W["l0.mix.k.b"] = torch.ones(32).to(torch.bfloat16)
    W["l0.mix.q.b"] = -torch.ones(64).to(torch.bfloat16)
    W["l0.mix.q.norm"] = W["l0.mix.k.norm"] = torch.ones(32)
    m = build(cfg, run, W=W)
    w, c, n = m.layers[0], m.cache, 60
    slot = c.alloc(n)
    c.extend([slot], [n])
    st = meta_for(c, slot, 0, n, run[0], chunk=50)
    rows = torch.zeros(n, w.wmix.shape[0], dtype=m.dtype, device=run[0])
    q = hops.talk_rows(rows, c.v[0], c.inv[0], st, w.talk, 1e-5)
    got = hops.talk_attn(q, c.v[0], c.inv[0], st, w.talk).cpu()[..., :32]
    seen = (torch.arange(n) % 50 + 1).double()
    e = seen * math.exp(9.0 * math.tanh(-32 * 0.5 / 9.0))
    want = (e / (1 + e))[:, None] * W["l0.mix.talk"].double().sum(1)
    assert float(errors(got, want[..., None].expand(n, 2, 32)).max()) < \
        (1e-4 if run[1] == "fp32" else 0.02)


@pytest.mark.parametrize("run", RUNS)
def test_rotation_far_out(run):
    """Queries at far positions, some of whose pairs are rotated."""
    n, dims, base = 6000, 12, 50.0
    cfg = config((attn(1, 1, 20, 4096, dims, base), None))
    m = build(cfg, run, max_seq=n)
    W, w, c, dev = weights_of(cfg), m.layers[0], m.cache, run[0]
    pos = torch.tensor([0, 1, 63, 64, 1000, 4095, 4096, 5999])
    rows = torch.randn(len(pos), 2, 64,
                       generator=torch.Generator().manual_seed(2))
    rows[..., 20:] = 0
    rows = rows.to(element(run))
    slot = c.alloc(n)
    c.extend([slot], [n])
    st = hops.StepMeta(nd=len(pos), pos=pos.to(dev, torch.int32),
                       slot=torch.full((len(pos),), slot, dtype=torch.int32,
                                       device=dev), table=c.table, max_len=n)
    got = hops.talk_rows(rows.flatten(1).to(dev), c.v[0], c.inv[0], st, w.talk,
                         1e-5)[:, 0, :20].cpu().double()
    order = _pair_order(20, dims)
    raw = torch.empty(len(pos), 20, dtype=torch.float64)
    raw[:, order] = rows[:, 0, :20].double()
    want = oracle.keys_of(raw + W["l0.mix.q.b"].double(),
                          W["l0.mix.q.norm"].double(), pos, base, dims, 1e-5)
    assert float((got - want[:, order]).abs().max()) < \
        (2e-5 if run[1] == "fp32" else 0.03)


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
    """Token by token from the first one on, over several pages and chunks."""
    cfg = config((attn(chunk=96), dense(64)), (attn(2, 1, chunk=50), None))
    m = build(cfg, run)
    ids = tokens(270, cfg, seed=4)
    slot = m.cache.alloc(0)
    close(feed(m, slot, ids, [1]), oracle.forward(cfg, weights_of(cfg), ids)[0],
          run)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("heads,kv,dim,chunk", [(24, 8, 32, 2000),
                                                (4, 1, 72, 700)])
def test_prompts_of_several_chunks_and_splits(heads, kv, dim, chunk, run):
    """Long spans: decoding splits its keys, also with the query's chunk just
    begun, and prompts take many tiles."""
    cfg = config((attn(heads, kv, dim, chunk, 16, scale=0.5), None))
    W = weights_of(cfg)
    m = build(cfg, run, W=W, max_seq=2200)
    ids = tokens(2100 if run[0] != "cpu" else 720, cfg, seed=7)
    cuts = [699, 1, 1, 1299, 1, 1, 17, 2, 1]
    slot, at, got, places = m.cache.alloc(0), 0, [], []
    for n in cuts:
        part = ids[at:at + n]
        if not part:
            break
        where = sorted({0, len(part) // 2, len(part) - 1})
        got.append(m.forward_step([(slot, part, where)]).cpu())
        places += [at + i for i in where]
        at += len(part)
    # one layer: its tokens' keys and values depend on the tokens alone
    close(torch.cat(got), one_layer_at(cfg, W, ids[:at], places), run, odd=0.1)


def one_layer_at(cfg, W, ids, places):
    """Logits of a model of one layer without a feed-forward, at some places."""
    W = {k: v.double() for k, v in W.items()}
    c, eps, gr = cfg["layers"][0]["mixer"], cfg["norm"]["eps"], \
        cfg["norm"]["groups"]
    x = W["embed"][torch.as_tensor(ids)]
    h = oracle.group_norm(x, W["l0.norm1"], gr, eps)
    H, G, d = c["heads"], c["kv_heads"], c["dim"]
    rot = (c["rot"]["base"], c["rot"]["dims"], eps)
    pos = torch.arange(len(ids))
    q = oracle.keys_of((h @ W["l0.mix.q"].T + W["l0.mix.q.b"]).view(-1, H, d),
                       W["l0.mix.q.norm"], pos, *rot)
    v = (h @ W["l0.mix.k"].T + W["l0.mix.k.b"]).view(-1, G, d)
    k = oracle.keys_of(v, W["l0.mix.k.norm"], pos, *rot)
    out = []
    for p in places:
        lo = p // c["mask"]["size"] * c["mask"]["size"]
        o = oracle.attend(q[p:p + 1], k[lo:p + 1], v[lo:p + 1],
                          W["l0.mix.talk"], c["scale"], c["softcap"], 10 ** 9)
        y = oracle.group_norm(o.reshape(1, -1) @ W["l0.mix.o"].T,
                              W["l0.norm1b"], gr, eps) * W["l0.ls1"]
        out.append(oracle.group_norm(x[p:p + 1] + y, W["final.norm"], gr, eps)
                   @ W["head"].T)
    return torch.cat(out)


@pytest.mark.parametrize("run", RUNS)
@pytest.mark.parametrize("heads", [4, 20, 40])
def test_many_rows_decode_at_once(heads, run):
    """Enough rows that no row's keys are split."""
    n = 290 if run[0] != "cpu" else 12
    cfg = config((attn(heads, 2, 16), dense()), (attn(chunk=64), None))
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
    spec = read_vivepel(FULL)
    assert spec.params == sum(v.numel() for v in W.values())
    assert [ly.mixer.chunk for ly in spec.layers] == [40, 100, 64, 7, 1000]
    assert spec.layers[1].ff is None and spec.norm_groups == 3
    m = HybridModel(spec, dtype="fp32", random_init=False)
    assert m.tensor_shapes() == {k: tuple(v.shape) for k, v in W.items()}
    assert ops_build.libs_of(spec) == ["hip", "hybrid", "talk"]
    assert ops_build.libs_of(get_spec("tiny-maferax")) == ["hip", "hybrid",
                                                           "latent"]
    assert ops_build.libs_of(get_spec("tiny")) == ["hip"]

    def broken(change):
        c = json.loads(json.dumps(FULL))
        change(c)
        with pytest.raises((ValueError, KeyError)):
            read_vivepel(c)

    broken(lambda c: c["norm"].pop("groups"))
    broken(lambda c: c["norm"].update(groups=5))
    broken(lambda c: c.update(window=3))
    broken(lambda c: c["layers"][1]["mixer"].pop("softcap"))
    broken(lambda c: c["layers"][1]["mixer"].update(softcap=0))
    broken(lambda c: c["layers"][1]["mixer"].update(vdim=41))
    broken(lambda c: c["layers"][1]["mixer"].update(kv_heads=2))
    broken(lambda c: c["layers"][0]["mixer"].update(window=4))
    broken(lambda c: c["layers"][0]["mixer"]["mask"].update(size=0))
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=15))
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=34))
    broken(lambda c: c["layers"][0].update(type="conv"))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="moe"))
    broken(lambda c: c["layers"][0]["mlp"].update(limit=7))


def test_values_alone_are_cached():
    spec = read_vivepel(FULL)
    m = HybridModel(spec, dtype="fp32", random_init=False, kv_tokens=256)
    assert all(k is None for k in m.cache.k)
    assert m.cache.bytes() == sum(
        5 * ly.mixer.kv_heads * 64 * (pd + 1) * 4
        for ly, pd in zip(spec.layers, (64, 64, 128, 64, 64)))


@pytest.fixture
def checkpoint(tmp_path):
    from safetensors.torch import save_file
    save_file(weights_of(FULL, 3), str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(FULL))
    return tmp_path


def test_checkpoint_describes_itself(checkpoint):
    spec = resolve_spec("llama3.2:1b", str(checkpoint))
    assert (spec.family, spec.name) == ("vivepel", "vivepel:custom")
    m = HybridModel(spec, dtype="fp32", random_init=False)
    assert m.load_safetensors(str(checkpoint)) == len(weights_of(FULL))
    from safetensors.torch import save_file
    W = weights_of(FULL, 3)
    del W["l2.ls2"]
    save_file(W, str(checkpoint / "model.safetensors"))
    with pytest.raises(KeyError, match="l2.ls2"):
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
@pytest.mark.parametrize("name", ["tiny-vivepel", "tiny-vivepel:latest"])
def test_registered_model_serves(name, run):
    eng = InferenceEngine(EngineConfig(model=name, device=run[0], dtype=run[1],
                                       max_batch_size=2, max_seq_len=128))
    r = eng.generate("hello", {"temperature": 0.7, "seed": 5,
                               "num_predict": 6})
    assert r.eval_count == 6
    assert "tiny-vivepel" in eng.model_names()
    info = eng.spec.model_info()
    assert info["general.architecture"] == "vivepel"
    assert info["vivepel.attention.chunk_size"] == 48


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_long_decode_by_captured_graphs(checkpoint, dtype):
    """Decode-only steps replay captured graphs, between eager mixed steps and
    synchronizations; every step against the eager model, 150 tokens long and
    over page and chunk borders."""
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
