"""Layer-list models: a decoder in which every layer names its mixer (softmax
attention over a paged cache, or mLSTM with a state per sequence) and its
feed-forward (dense gated, or routed experts).

One step function serves prompts, portions of prompts and decoding, also mixed
in one batch: `forward_step`. Its tokens are ordered decode rows first, so each
mixer runs its decode kernels on the head of the batch and its prefill kernels
on the rest while projections, experts and norms see one matrix.
`forward_decode` is the same with decode rows only, driven by device tensors
alone so that it can be captured in a hipGraph.

Layout: widths, head sizes and feed-forward sizes are padded to multiples of 64
with zero weights at load, so kernels need no edge handling and the padding
carries zeros all the way. The residual stream is f32; the activations and
weights are bf16, or f32 in the exact mode (dtype "fp32"), which runs on the
GPU too.
"""

from __future__ import annotations

import glob
import os
from dataclasses import dataclass
from typing import Callable, Optional, Sequence

import numpy as np
import torch

from gridllm_amd.models.paged import PagedCache, head_pad, pad64
from gridllm_amd.models.registry import (AttentionMixer, DenseFF, HybridSpec,
                                         RoutedFF)
from gridllm_amd.ops import hybrid as hops
from gridllm_amd.ops.autotune import linear as _linear
from gridllm_amd.ops.autotune import linear_gateup as _linear_gateup
from gridllm_amd.ops.hybrid import StepMeta
from gridllm_amd.ops.reference import Glu
from gridllm_amd.parallel.tp import TPContext

_DTYPES = {"bf16": torch.bfloat16, "fp32": torch.float32}
_NORM_OFFSET = 1.0              # norm weights are stored around zero


@dataclass
class BlockWeights:
    """One layer's tensors, fused and padded. Dense: gateup and down are 2-D;
    routed: up [E, F, W], down [E, W, F]."""
    wmix: torch.Tensor                    # q, k, v, output gate
    wo: torch.Tensor
    norm1: torch.Tensor
    norm2: Optional[torch.Tensor] = None
    sink: Optional[torch.Tensor] = None
    wgates: Optional[torch.Tensor] = None     # input and forget gate rows
    bgates: Optional[torch.Tensor] = None
    mnorm: Optional[torch.Tensor] = None
    wgateup: Optional[torch.Tensor] = None
    up: Optional[torch.Tensor] = None
    down: Optional[torch.Tensor] = None
    router: Optional[torch.Tensor] = None


def _pad(t: torch.Tensor, *shape: int) -> torch.Tensor:
    """t in the corner of zeros of `shape`."""
    if tuple(t.shape) == shape:
        return t
    out = t.new_zeros(shape)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


def _pad_heads(t: torch.Tensor, heads: int, to: int) -> torch.Tensor:
    """Rows [heads * d, ...] -> [heads * to, ...], zero rows behind each head."""
    d = t.shape[0] // heads
    t = t.view(heads, d, *t.shape[1:])
    return _pad(t, heads, to, *t.shape[2:]).reshape(heads * to, *t.shape[2:])


class HybridModel:
    supports_mixed = True          # portions of prompts beside decoded tokens
    supports_shift = False         # learned positions and states cannot slide

    def __init__(self, spec: HybridSpec, device: str = "cpu",
                 dtype: str = "bf16", tp: Optional[TPContext] = None,
                 seed: int = 0, kv_slots: int = 64, max_seq: int = 0,
                 kv_tokens: int = 0, random_init: bool = True):
        if tp is not None and tp.size > 1:
            raise NotImplementedError("layer-list models run on one GPU")
        if dtype not in _DTYPES:
            raise ValueError(f"layer-list models run in bf16 or fp32, "
                             f"not {dtype}")
        self.spec = spec
        self.tp = tp or TPContext()
        self.device = torch.device(device)
        self.dtype = _DTYPES[dtype]
        self.max_seq = min(max_seq or spec.max_seq_len, spec.positions)
        if kv_tokens:                      # one sequence has to fit the pool
            self.max_seq = min(self.max_seq, pad64(kv_tokens))
        self.rope_len = self.max_seq       # bound of positions
        self.width = pad64(spec.hidden)
        if self.width > 8192:
            raise ValueError(f"width {spec.hidden}: more than 8192")
        self.gateup_il = False
        from gridllm_amd.utils.pinned import PinnedUploader
        self.up = PinnedUploader(self.device)
        self.cache = PagedCache(spec, kv_slots, self.max_seq, self.device,
                                self.dtype, pool_tokens=kv_tokens,
                                upload=self.up.upload)
        if random_init:
            self._init_weights(seed)

    # -- weights -----------------------------------------------------------

    def tensor_shapes(self) -> dict[str, tuple]:
        """Name and shape of every tensor a checkpoint of the spec holds."""
        s = self.spec
        w = s.hidden
        out = {"embed": (s.vocab, w), "pos": (s.positions, w),
               "final.norm": (w,)}
        for i, ly in enumerate(s.layers):
            if ly.weights_of is not None:
                continue
            p, mx, ff = f"l{i}.", ly.mixer, ly.ff
            h = mx.heads
            attn = isinstance(mx, AttentionMixer)
            kv = mx.kv_heads if attn else h
            out |= {p + "norm1": (w,), p + "mix.q": (h * mx.dim, w),
                    p + "mix.k": (kv * mx.dim, w),
                    p + "mix.v": (kv * mx.vdim, w),
                    p + "mix.o": (w, h * mx.vdim)}
            if attn:
                out |= {p + "mix.sink": (h,), p + "mix.g": (h, w)}
            else:
                out |= {p + "mix.g": (h * mx.vdim, w),
                        p + "mix.norm": (h * mx.vdim,),
                        p + "mix.i": (h, w), p + "mix.i.b": (h,),
                        p + "mix.f": (h, w), p + "mix.f.b": (h,)}
            if ff is None:
                continue
            out[p + "norm2"] = (w,)
            if isinstance(ff, DenseFF):
                out |= {p + "mlp.gate": (ff.ff, w), p + "mlp.up": (ff.ff, w),
                        p + "mlp.down": (w, ff.ff)}
            else:
                out[p + "mlp.router"] = (ff.experts, w)
                for e in range(ff.experts):
                    out |= {f"{p}mlp.e{e}.up": (ff.ff, w),
                            f"{p}mlp.e{e}.down": (w, ff.ff)}
        return out

    def _init_weights(self, seed: int) -> None:
        """Random init: projections at the usual 0.02, norms and gates near
        their neutral values. Drawn tensor by tensor while the layers are
        built, so a large model never exists twice."""
        gen = torch.Generator(device=self.device)
        gen.manual_seed(seed or 1234)
        shapes = self.tensor_shapes()

        def draw(name: str) -> torch.Tensor:
            sh = shapes[name]
            if name.endswith("mix.norm"):
                return torch.ones(sh, device=self.device)
            if name.endswith(".norm1") or name.endswith(".norm2") or \
                    name.endswith(".norm") or name.endswith("i.b"):
                return torch.zeros(sh, device=self.device)
            if name.endswith("f.b"):
                return torch.full(sh, 4.0, device=self.device)
            return torch.randn(sh, generator=gen, device=self.device) * 0.02

        self._assemble(draw)

    def load_safetensors(self, path: str) -> int:
        """Load a checkpoint folder by tensor name; returns the number of
        tensors used. Missing tensors and wrong shapes raise."""
        from safetensors import safe_open
        files = sorted(glob.glob(os.path.join(path, "*.safetensors")))
        if not files:
            raise FileNotFoundError(f"no .safetensors under {path!r}")
        want = self.tensor_shapes()
        where = {}
        handles = [safe_open(f, framework="pt") for f in files]
        for sf in handles:
            for k in sf.keys():
                where[k] = sf
        missing = sorted(set(want) - set(where))
        if missing:
            raise KeyError(f"missing weights: {missing[:5]} "
                           f"(+{max(0, len(missing) - 5)} more)")

        def read(name: str) -> torch.Tensor:
            t = where[name].get_tensor(name)
            if tuple(t.shape) != want[name]:
                raise ValueError(f"{name}: {tuple(t.shape)}, the config "
                                 f"gives {want[name]}")
            return t.to(self.device)

        self._assemble(read)
        return len(want)

    def _assemble(self, get: Callable[[str], torch.Tensor]) -> None:
        """Build the fused, padded layout from tensors by name."""
        s, wp = self.spec, self.width
        self.gateup_il = False

        def mat(t, rows=None):          # [out, in] -> element type, padded in
            return _pad(t.to(self.dtype), rows or t.shape[0], pad64(t.shape[1]))

        def vec(t, n):
            return _pad(t.float(), n)

        self.embed = mat(get("embed"))
        self.pos_table = mat(get("pos"))
        self.final_norm = vec(get("final.norm"), wp)
        built: dict[int, BlockWeights] = {}
        for i, ly in enumerate(s.layers):
            if ly.weights_of is None:
                built[i] = self._assemble_layer(f"l{i}.", ly, get, mat, vec)
        self.layers = [built[s.owner(i)] for i in range(len(s.layers))]

    def _assemble_layer(self, p: str, ly, get, mat, vec) -> BlockWeights:
        mx, ff, wp = ly.mixer, ly.ff, self.width
        h = mx.heads
        attn = isinstance(mx, AttentionMixer)
        kv = mx.kv_heads if attn else h
        dk = head_pad(mx) if attn else pad64(mx.dim)
        dv = dk if attn else pad64(mx.vdim)
        g = mat(get(p + "mix.g"))
        parts = [_pad_heads(mat(get(p + "mix.q")), h, dk),
                 _pad_heads(mat(get(p + "mix.k")), kv, dk),
                 _pad_heads(mat(get(p + "mix.v")), kv, dv),
                 g if attn else _pad_heads(g, h, dv)]
        wmix = torch.cat(parts)
        wmix = _pad(wmix, -(-wmix.shape[0] // 128) * 128, wp).contiguous()
        # columns of the output projection follow the padded heads
        wo = _pad_heads(get(p + "mix.o").to(self.dtype).T, h, dv).T
        w = BlockWeights(
            wmix=wmix, wo=_pad(wo, wp, h * dv).contiguous(),
            norm1=vec(get(p + "norm1"), wp))
        if attn:
            w.sink = get(p + "mix.sink").float()
        else:
            w.wgates = torch.cat([mat(get(p + "mix.i")),
                                  mat(get(p + "mix.f"))]).contiguous()
            w.bgates = torch.cat([get(p + "mix.i.b"),
                                  get(p + "mix.f.b")]).float()
            w.mnorm = _pad_heads(get(p + "mix.norm").float(), h, dv)
        if ff is None:
            return w
        w.norm2 = vec(get(p + "norm2"), wp)
        fp = pad64(ff.ff)
        if isinstance(ff, DenseFF):
            w.wgateup = torch.cat([mat(get(p + "mlp.gate"), fp),
                                   mat(get(p + "mlp.up"), fp)])
            w.down = mat(get(p + "mlp.down"), wp)
            return w
        w.router = mat(get(p + "mlp.router"))
        w.up = torch.empty(ff.experts, fp, wp, dtype=self.dtype,
                           device=self.device)
        w.down = torch.empty(ff.experts, wp, fp, dtype=self.dtype,
                             device=self.device)
        for e in range(ff.experts):
            w.up[e] = mat(get(f"{p}mlp.e{e}.up"), fp)
            w.down[e] = mat(get(f"{p}mlp.e{e}.down"), wp)
        return w

    def unique_layers(self) -> list[BlockWeights]:
        return list({id(w): w for w in self.layers}.values())

    def gemm_shapes(self) -> tuple[list, list]:
        """(n, k) of the decode projections, and of the gate/up ones."""
        plain = {tuple(self.embed.shape)}
        gu = set()
        for w in self.unique_layers():
            plain |= {tuple(w.wmix.shape), tuple(w.wo.shape)}
            if w.wgateup is not None:
                gu.add(tuple(w.wgateup.shape))
                plain.add(tuple(w.down.shape))
        return sorted(plain), sorted(gu)

    def interleave_gateup(self) -> None:
        """Gate and up rows in groups of 64 | 64, the layout of the fused
        gate/up projection (as LlamaModel.interleave_gateup)."""
        if self.gateup_il:
            return
        for w in self.unique_layers():
            if w.wgateup is not None:
                n, k = w.wgateup.shape
                w.wgateup = w.wgateup.view(2, n // 128, 64, k).transpose(
                    0, 1).reshape(n, k).contiguous()
        self.gateup_il = True

    def param_bytes(self) -> int:
        ts = [self.embed, self.pos_table, self.final_norm]
        for w in self.unique_layers():
            ts += [t for t in vars(w).values() if t is not None]
        return sum(t.numel() * t.element_size() for t in ts)

    # -- layers ------------------------------------------------------------

    def _mix(self, i: int, w: BlockWeights, mx, xb: torch.Tensor,
             st: StepMeta) -> torch.Tensor:
        c, eps = self.cache, self.spec.norm_eps
        rows = _linear(xb, w.wmix)
        if isinstance(mx, AttentionMixer):
            h, g, p = mx.heads, mx.kv_heads, c.k[i].shape[3]
            q = hops.qknorm_kv(rows, c.k[i], c.v[i], st, h, g, mx.dim, eps,
                               mx.q_coef, mx.q_every)
            gate = rows[:, (h + 2 * g) * p:(h + 2 * g) * p + h]
            o = hops.paged_attn(q, c.k[i], c.v[i], st, mx.scale, w.sink,
                                gate).view(xb.shape[0], -1)
        else:
            gates = hops.proj_f32(xb, w.wgates, w.bgates)
            o = hops.mlstm(rows, gates, c.S[i], c.m[i], w.mnorm, st, mx.dim,
                           mx.vdim, mx.gate_cap, eps)
        return _linear(o, w.wo)

    def _feed(self, w: BlockWeights, ff, xb: torch.Tensor):
        """Feed-forward output, and the pair weights if it is still a row per
        (token, chosen expert)."""
        if isinstance(ff, DenseFF):
            glu = Glu(ff.alpha, ff.limit, ff.shift)
            act = _linear_gateup(xb, w.wgateup, glu) if self.gateup_il else \
                hops.glu(_linear(xb, w.wgateup), glu)
            return _linear(act, w.down), None
        assert isinstance(ff, RoutedFF)
        return hops.moe(xb, hops.proj_f32(xb, w.router), w.up, w.down, ff.top)

    def _run(self, tokens: torch.Tensor, st: StepMeta,
             trail: Optional[list] = None) -> torch.Tensor:
        """The residual stream behind the last layer, f32 [n, W]; trail
        collects it behind every layer."""
        s = self.spec
        x, xb = hops.embed_pos(tokens, st.pos, self.embed, self.pos_table)
        for i, (ly, w) in enumerate(zip(s.layers, self.layers)):
            y = self._mix(i, w, ly.mixer, xb, st)
            hops.post_norm(x, xb, y, w.norm1, _NORM_OFFSET, s.hidden,
                           s.norm_eps)
            if ly.ff is not None:
                y, pair_w = self._feed(w, ly.ff, xb)
                hops.post_norm(x, xb, y, w.norm2, _NORM_OFFSET, s.hidden,
                               s.norm_eps, pair_w)
            if trail is not None:
                trail.append(x[:, :s.hidden].clone())
        return x

    def _head(self, x: torch.Tensor, rows: Optional[torch.Tensor]
              ) -> torch.Tensor:
        h = hops.norm_rows(x, rows, self.final_norm, _NORM_OFFSET,
                           self.spec.hidden, self.spec.norm_eps, self.dtype)
        return _linear(h, self.embed).float()

    # -- steps -------------------------------------------------------------

    @torch.no_grad()
    def forward_step(self, entries: Sequence[tuple], return_hidden=False,
                     trail: Optional[list] = None):
        """One batch of (slot, token ids, wanted places): each entry's tokens
        continue its slot's sequence. Returns logits f32 [wanted, vocab], in
        the order of the entries and of their places; with return_hidden, also
        the mean of each entry's normed final states [entries, hidden]."""
        for _, ids, want in entries:
            if not len(ids) or any(not 0 <= w < len(ids) for w in want):
                raise ValueError("an entry without tokens, or a place "
                                 "outside of it")
        if len({e[0] for e in entries}) != len(entries):
            raise ValueError("a sequence twice in one step")
        order = sorted(range(len(entries)),
                       key=lambda i: len(entries[i][1]) > 1)
        starts = [int(self.cache.lens[e[0]]) for e in entries]
        self.cache.extend([e[0] for e in entries],
                          [len(e[1]) for e in entries])
        off, first = 0, {}
        toks, pos, slot = [], [], []
        segs, tiles, chunks, csegs = [], [], [], []
        nd = 0
        for i in order:
            sl, ids, _ = entries[i]
            ln, p0 = len(ids), starts[i]
            first[i] = off
            toks.append(np.asarray(ids, dtype=np.int64))
            pos.append(np.arange(p0, p0 + ln))
            slot.append(np.full(ln, sl))
            segs.append((off, ln, sl, p0))
            if ln == 1:
                nd += 1
            else:
                tiles += [(off, ln, sl, q0, p0, 0, 0, 0)
                          for q0 in range(0, ln, 128)]
                csegs.append((sl, p0, len(chunks), -(-ln // 64)))
                chunks += [(off + c, min(64, ln - c), len(csegs) - 1, 0)
                           for c in range(0, ln, 64)]
            off += ln
        ids_np = np.concatenate(toks)
        if ids_np.min() < 0 or ids_np.max() >= self.spec.vocab:
            raise ValueError("token id outside of the vocabulary")
        want = [first[i] + w for i, e in enumerate(entries) for w in e[2]]
        tokens = self.up.upload(ids_np)
        parts = [np.concatenate(pos), np.concatenate(slot), np.asarray(want),
                 np.asarray(segs), np.asarray(tiles), np.asarray(chunks),
                 np.asarray(csegs)]
        dev = self._upload_ints(parts)
        mixed = bool(tiles)
        st = StepMeta(nd=nd, pos=dev[0], slot=dev[1], table=self.cache.table,
                      max_len=self.max_seq,
                      segs=dev[3].view(-1, 4) if mixed else None,
                      tiles=dev[4].view(-1, 8) if mixed else None,
                      chunks=dev[5].view(-1, 4) if mixed else None,
                      chunk_segs=dev[6].view(-1, 4) if mixed else None)
        x = self._run(tokens, st, trail)
        ends = np.asarray([[e[0] for e in entries],
                           [p + len(e[1]) for p, e in zip(starts, entries)]],
                          dtype=np.int64)
        ends = self.up.upload(ends)
        self.cache.seq_lens.index_copy_(0, ends[0], ends[1].to(torch.int32))
        logits = self._head(x, dev[2]) if want else \
            torch.empty(0, self.spec.vocab, device=self.device)
        if not return_hidden:
            return logits
        h = hops.norm_rows(x, None, self.final_norm, _NORM_OFFSET,
                           self.spec.hidden, self.spec.norm_eps, self.dtype)
        h = h[:, :self.spec.hidden].float()
        return logits, torch.stack(
            [h[first[i]:first[i] + len(e[1])].mean(0)
             for i, e in enumerate(entries)])

    def _upload_ints(self, parts: list) -> list[torch.Tensor]:
        """int32 arrays to the device in one copy; each starts at a multiple
        of 4 elements (kernels read some as int4)."""
        flat, at = [], []
        n = 0
        for a in parts:
            a = np.asarray(a, dtype=np.int32).reshape(-1)
            at.append((n, a.size))
            pad = -a.size % 4
            flat += [a, np.zeros(pad, dtype=np.int32)]
            n += a.size + pad
        dev = self.up.upload(np.concatenate(flat))
        return [dev[o:o + c] for o, c in at]

    def forward_prefill(self, tokens: torch.Tensor, slot: int,
                        start_pos: int = 0, return_hidden: bool = False):
        """One sequence's tokens from start_pos on; logits of the last one."""
        if start_pos != self.cache.lens[slot]:
            raise ValueError(f"slot {slot} holds {self.cache.lens[slot]} "
                             f"tokens, not {start_pos}")
        ids = tokens.tolist()
        out = self.forward_step([(slot, ids, [len(ids) - 1])], return_hidden)
        return (out[0][0], out[1][0]) if return_hidden else out[0]

    def forward_prefill_batch(self, token_lists: list, slots: list,
                              return_hidden: bool = False):
        """Several fresh sequences in one step; logits of each last token."""
        lists = [t.tolist() for t in token_lists]
        return self.forward_step(
            [(sl, ids, [len(ids) - 1]) for sl, ids in zip(slots, lists)],
            return_hidden)

    @torch.no_grad()
    def forward_decode(self, tokens: torch.Tensor,
                       slot_map: torch.Tensor) -> torch.Tensor:
        """One decode step of a batch, from device tensors alone (capturable):
        tokens [B] int64, slot_map [B] int32 -> logits f32 [B, vocab]. The
        cache must have been prepared for the slots (prepare_decode)."""
        slots = slot_map.long()
        st = StepMeta(nd=tokens.shape[0], pos=self.cache.seq_lens[slots],
                      slot=slot_map, table=self.cache.table,
                      max_len=self.max_seq)
        x = self._run(tokens, st)
        self.cache.seq_lens.index_add_(
            0, slots, torch.ones_like(slot_map))
        return self._head(x, None)
