"""What the tests of the layer-list models share: devices and tolerances,
feeding a model in portions, steps laid out by hand, prompts as bytes."""

import os

import pytest
import torch

from gridllm_amd.ops.hybrid import ChunkPortions, StepMeta

REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
RUNS = [pytest.param(("cpu", "fp32"), id="cpu"),
        pytest.param(("cuda:0", "fp32"), id="gpu-f32", marks=pytest.mark.gpu),
        pytest.param(("cuda:0", "bf16"), id="gpu-bf16", marks=pytest.mark.gpu)]
EXACT = RUNS[:2]


@pytest.fixture(autouse=True)
def one_thread():
    """Thousands of tiny CPU products: threads only get in their way."""
    n = torch.get_num_threads()
    torch.set_num_threads(1)
    yield
    torch.set_num_threads(n)


def feed(m, slot, ids, sizes):
    """Run ids in portions of `sizes` (the last one repeats); all logits."""
    out, at, k = [], 0, 0
    while at < len(ids):
        n = sizes[min(k, len(sizes) - 1)]
        part = ids[at:at + n]
        out.append(m.forward_step([(slot, part, list(range(len(part))))]))
        at, k = at + len(part), k + 1
    return torch.cat(out).cpu()


def whole(m, ids):
    slot = m.cache.alloc(0)
    out = feed(m, slot, ids, [len(ids)])
    m.cache.free(slot)
    return out


def errors(got, want):
    """Per row: rms difference over the row's own rms."""
    want = want.to(torch.float64)
    d = got.cpu().to(torch.float64) - want
    return (d.pow(2).mean(-1) / want.pow(2).mean(-1)).sqrt()


def close(got, want, run, exact=2e-4, coarse=0.04, odd=0.04):
    """f32: every row. bf16: all but a few rows in which a close call of the
    router went the other way."""
    e = errors(got, want)
    if run[1] == "fp32":
        assert float(e.max()) < exact, float(e.max())
    else:
        bad = int((e > coarse).sum())
        assert bad <= odd * len(e), (bad, len(e), float(e.max()))


def meta_for(cache, slot, start, ln, dev, absorb=16, chunk=0):
    """Step of one entry, as forward_step lays it out. Latent and talking-heads
    attention take portions of up to `absorb` tokens one by one; `chunk` is the
    latter's."""
    def t(a, w):
        return torch.tensor(a, dtype=torch.int32, device=dev).view(-1, w)
    st = StepMeta(nd=1 if ln == 1 else 0,
                  pos=torch.arange(start, start + ln, dtype=torch.int32,
                                   device=dev),
                  slot=torch.full((ln,), slot, dtype=torch.int32, device=dev),
                  table=cache.table, max_len=cache.max_seq)
    if ln > 1:
        st.segs = t([[0, ln, slot, start]], 4)
        st.tiles = t([[0, ln, slot, q, start, 0, 0, 0]
                      for q in range(0, ln, 128)], 8)
        st.chunks = t([[c, min(64, ln - c), 0, 0]
                       for c in range(0, ln, 64)], 4)
        st.chunk_segs = t([[slot, start, 0, -(-ln // 64)]], 4)
    if ln <= absorb:
        st.absorbed = ln
    else:
        total = start + ln
        st.lat_rows = -(-total // 32) * 32
        st.lat_items = t([[c // 64, slot, c, min(64, total - c) + 256 * min(
            64, st.lat_rows - c)] for c in range(0, total, 64)], 4)
        st.lat_tiles = t([[0, ln, 0, q, start, 0, 0, 0]
                          for q in range(0, ln, 128)], 8)
        if chunk:
            p0 = start // chunk * chunk // 64          # first page seen
            n = -(-total // 64) - p0
            st.talk[chunk] = ChunkPortions(
                n, min(total, chunk),
                t([[p0 + i, slot, i, min(64, total - 64 * (p0 + i))]
                   for i in range(n)], 4),
                *(t([[0, ln, 0, q, start, p0, 0, 0]
                     for q in range(0, ln, k)], 8) for k in (16, 128)))
    return st


def portions(n, how):
    cuts, at = [], 0
    while at < n:
        ln = min(how[min(len(cuts), len(how) - 1)], n - at)
        cuts.append((at, ln))
        at += ln
    return cuts


class Bytes:
    """Prompts as bytes; every id decodes to something, none ends a text."""
    eos_id = -1

    def __init__(self, vocab):
        self.vocab = vocab

    def encode(self, text):
        return [b % self.vocab for b in text.encode()]

    def decode(self, ids):
        return "".join(chr(33 + i % 90) for i in ids)

    def decode_stream(self):
        tok = self

        class D:
            def push(self, i):
                return tok.decode([i])
        return D()
