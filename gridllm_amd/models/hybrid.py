"""Layer-list models: a decoder in which every layer names its mixer (softmax,
latent or talking-heads attention over a paged cache, mLSTM, gated linear or
lightning attention with a state per sequence, or attention and a recurrence
side by side) and its feed-forward (dense gated, dense with PolyNorm, or routed
experts, with or without a shared one).

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

from gridllm_amd.models.paged import (PAGE, PagedCache, head_pad, latent_pad,
                                      pad64, rotated_pad)
from gridllm_amd.models.registry import (AttentionMixer, DenseFF, GlaMixer,
                                         HybridSpec, LatentMixer,
                                         LightningMixer, ParallelMixer, PolyFF,
                                         Rotary, RoutedFF, TalkingMixer)
from gridllm_amd.ops import hybrid as hops
from gridllm_amd.ops.autotune import linear as _linear
from gridllm_amd.ops.autotune import linear_gateup as _linear_gateup
from gridllm_amd.ops.hybrid import (ChunkPortions, Choice, DepthAverage, Keys,
                                    StepMeta, Talk)
from gridllm_amd.ops.reference import SWIGLU, Glu
from gridllm_amd.parallel.tp import TPContext

_DTYPES = {"bf16": torch.bfloat16, "fp32": torch.float32}
# portions of up to this many tokens run latent and talking-heads attention
# token by token against the cached rows; for longer ones it pays to lay out
# keys and values
_ABSORB = 16


@dataclass
class BlockWeights:
    """One layer's tensors, fused and padded. Dense: gateup and down are 2-D;
    routed: up [E, F, W] (gated: [E, 2 F, W], rows in turns of 16 gate | 16
    up), down [E, W, F]; gateup and sdown are the shared expert's, and the last
    row of router is its gate's."""
    wmix: torch.Tensor                    # q, k, v, output gate; or the
                                          # projections to latents, gate
    wo: torch.Tensor
    norm1: torch.Tensor
    norm2: Optional[torch.Tensor] = None
    sink: Optional[torch.Tensor] = None
    wgates: Optional[torch.Tensor] = None     # input and forget gate rows
    bgates: Optional[torch.Tensor] = None
    mnorm: Optional[torch.Tensor] = None
    qnorm: Optional[torch.Tensor] = None      # latent attention
    kvnorm: Optional[torch.Tensor] = None
    wuq: Optional[torch.Tensor] = None
    wuk: Optional[torch.Tensor] = None        # [H, KR, P]
    wuv: Optional[torch.Tensor] = None        # [H, P, KR]
    wukv: Optional[torch.Tensor] = None       # [H, 2 P, KR]
    wa2: Optional[torch.Tensor] = None        # decays: [rank, H * DK]
    ba2: Optional[torch.Tensor] = None
    talk: Optional[Talk] = None               # talking-heads attention
    act: Optional[torch.Tensor] = None        # PolyNorm's numbers
    pre1: Optional[torch.Tensor] = None       # norms ahead of the sublayers
    pre2: Optional[torch.Tensor] = None
    decay: Optional[torch.Tensor] = None      # by head: decays, logarithms
    hc1: Optional[torch.Tensor] = None        # streams: mix, then put
    hc2: Optional[torch.Tensor] = None
    read1: Optional[torch.Tensor] = None      # weights of what is read
    read2: Optional[torch.Tensor] = None
    corr: Optional[torch.Tensor] = None
    avg: Optional[torch.Tensor] = None        # depth average
    wgateup: Optional[torch.Tensor] = None
    up: Optional[torch.Tensor] = None
    down: Optional[torch.Tensor] = None
    sdown: Optional[torch.Tensor] = None
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


def _pair_order(dim: int, rot_dims: int) -> torch.Tensor:
    """Coordinates of a head such that the pairs (i, i + rot_dims / 2) become
    neighbours, in front."""
    i = torch.arange(rot_dims // 2)
    pairs = torch.stack([i, i + rot_dims // 2], dim=1).flatten()
    return torch.cat([pairs, torch.arange(rot_dims, dim)])


def _glu(ff: Optional[DenseFF]) -> Glu:
    return SWIGLU if ff is None else Glu(ff.alpha, ff.limit, ff.shift,
                                         ff.cubic)


class HybridModel:
    supports_mixed = True          # portions of prompts beside decoded tokens
    supports_shift = False         # states and pages cannot slide

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
        self.max_seq = max_seq or spec.max_seq_len
        if spec.positions:
            self.max_seq = min(self.max_seq, spec.positions)
        elif kv_tokens and not max_seq:    # nothing but the pool bounds it
            self.max_seq = pad64(kv_tokens)
        if kv_tokens:                      # one sequence has to fit the pool
            self.max_seq = min(self.max_seq, pad64(kv_tokens))
        self.norm_off = 0.0 if spec.scalar_norms or spec.plain_norms else 1.0
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
        self.rot = self._rotations()
        mixers = [ly.mixer for ly in spec.layers]
        # latents of prompt portions are expanded; keys within these chunk
        # sizes laid out
        self.expands = dtype == "bf16" and any(
            isinstance(m, LatentMixer) for m in mixers)
        self.chunks = sorted({m.chunk for m in mixers
                              if isinstance(m, TalkingMixer)}) \
            if dtype == "bf16" else []
        if random_init:
            self._init_weights(seed)

    def _rotations(self) -> list[Optional[tuple]]:
        """Per layer with rotated queries and keys, cos and sin of position
        times frequency, f32 [rows, R / 2] for the positions of whole pages; 1
        and 0 for pairs that are not rotated."""
        rows = pad64(self.max_seq)
        made: dict[tuple, tuple] = {}

        def table(mx) -> Optional[tuple]:
            if isinstance(mx, AttentionMixer):
                rot = mx.rot
                r = -(-rot.dims // 8) * 8 if rot else 0
            elif mx is not None:
                rot = Rotary(mx.rot_base, mx.rot_dims)
                r = latent_pad(mx)[1] if isinstance(mx, LatentMixer) else \
                    rotated_pad(mx)
            if mx is None or rot is None:
                return None
            if (rot, r) not in made:
                f, grow = rot.frequencies()
                half = len(f)
                a = torch.outer(torch.arange(rows, dtype=torch.float64),
                                torch.tensor(f, dtype=torch.float64))
                cos = torch.ones(rows, r // 2, dtype=torch.float64)
                sin = torch.zeros_like(cos)
                cos[:, :half], sin[:, :half] = a.cos() * grow, a.sin() * grow
                made[rot, r] = tuple(t.float().to(self.device).contiguous()
                                     for t in (cos, sin))
            return made[rot, r]

        return [table(ly.attention()) for ly in self.spec.layers]

    # -- weights -----------------------------------------------------------

    def tensor_shapes(self) -> dict[str, tuple]:
        """Name and shape of every tensor a checkpoint of the spec holds."""
        s = self.spec
        w = s.hidden
        norm = () if s.scalar_norms else (w,)
        out = {"embed": (s.vocab, w), "final.norm": norm}
        if s.positions:
            out["pos"] = (s.positions, w)
        if s.embed_norm:
            out["embed.norm"] = norm
        if not s.tied:
            out["head"] = (s.vocab, w)
        for i, ly in enumerate(s.layers):
            if s.depth_average:
                out[f"l{i}.dwa"] = (i + 2,)
            if ly.weights_of is not None:
                continue
            p, mx, ff = f"l{s.number(i)}.", ly.mixer, ly.ff
            out |= self._mixer_shapes(p + "mix.", mx)
            for k in (1, 2) if ff is not None else (1,):
                out[f"{p}norm{k}"] = norm
                if s.streams:
                    out |= {f"{p}hc{k}.in": (s.streams,),
                            f"{p}hc{k}.out": (s.streams,),
                            f"{p}hc{k}.mix": (s.streams, s.streams)}
                if s.pre_norms:
                    out[f"{p}norm{k}b"] = norm
                if s.layer_scale:
                    out[f"{p}ls{k}"] = (w,)
            if ff is None:
                continue
            if isinstance(ff, PolyFF):
                out |= {p + "mlp.up": (ff.ff, w), p + "mlp.down": (w, ff.ff),
                        p + "mlp.act": (4,)}
                continue
            if isinstance(ff, DenseFF):
                out |= {p + "mlp.gate": (ff.ff, w), p + "mlp.up": (ff.ff, w),
                        p + "mlp.down": (w, ff.ff)}
                continue
            out[p + "mlp.router"] = (ff.outputs, w)
            if ff.corrected:
                out[p + "mlp.correction"] = (ff.outputs,)
            for e in range(ff.experts):
                out |= {f"{p}mlp.e{e}.up": (ff.ff, w),
                        f"{p}mlp.e{e}.down": (w, ff.ff)}
                if ff.gated:
                    out[f"{p}mlp.e{e}.gate"] = (ff.ff, w)
            if ff.shared is not None:
                out |= {p + "mlp.shared.gate": (ff.shared.ff, w),
                        p + "mlp.shared.up": (ff.shared.ff, w),
                        p + "mlp.shared.down": (w, ff.shared.ff),
                        p + "mlp.shared.sg": (1, w)}
        return out

    def _mixer_shapes(self, p: str, mx) -> dict[str, tuple]:
        if isinstance(mx, ParallelMixer):
            return self._mixer_shapes(p + "left.", mx.left) | \
                self._mixer_shapes(p + "right.", mx.right)
        w, h = self.spec.hidden, mx.heads
        if isinstance(mx, LatentMixer):
            qr, k = mx.q_rank, mx.kv_rank
            return {p + "dq": (qr, w), p + "dq.norm": (qr,),
                    p + "uq": (h * (mx.dim + mx.rot_dim), qr),
                    p + "dkv": (k + mx.rot_dim, w), p + "dkv.norm": (k,),
                    p + "uk": (h * mx.dim, k), p + "uv": (h * mx.vdim, k),
                    p + "g": (h, w), p + "o": (w, h * mx.vdim)}
        if isinstance(mx, TalkingMixer):
            q, k = h * mx.dim, mx.kv_heads * mx.dim
            return {p + "q": (q, w), p + "q.b": (q,), p + "k": (k, w),
                    p + "k.b": (k,), p + "q.norm": (mx.dim,),
                    p + "k.norm": (mx.dim,), p + "talk": (h, h),
                    p + "o": (w, q)}
        attn = isinstance(mx, AttentionMixer)
        kv = mx.kv_heads if attn else h
        out = {p + "q": (h * mx.dim, w), p + "k": (kv * mx.dim, w),
               p + "v": (kv * mx.vdim, w), p + "o": (w, h * mx.vdim)}
        if attn:
            if mx.sink:
                out[p + "sink"] = (h,)
            gates = h * mx.vdim if mx.gate == "element" else h
            return out | {p + "g": (gates, w)}
        out[p + "g"] = (h * mx.vdim, w)
        if isinstance(mx, LightningMixer):
            return out | {p + "norm": (h * mx.vdim,)}
        if isinstance(mx, GlaMixer):
            return out | {p + "norm": (mx.vdim,), p + "a1": (mx.rank, w),
                          p + "a2": (h * mx.dim, mx.rank),
                          p + "a2.b": (h * mx.dim,)}
        return out | {p + "norm": (h * mx.vdim,), p + "i": (h, w),
                      p + "i.b": (h,), p + "f": (h, w), p + "f.b": (h,)}

    def _init_weights(self, seed: int) -> None:
        """Random init: projections at the usual 0.02, norms and gates near
        their neutral values. Drawn tensor by tensor while the layers are
        built, so a large model never exists twice."""
        gen = torch.Generator(device=self.device)
        gen.manual_seed(seed or 1234)
        shapes = self.tensor_shapes()

        def draw(name: str) -> torch.Tensor:
            sh, last = shapes[name], name.rsplit(".", 1)[-1]
            if last == "dwa":              # mostly the layer's own result
                t = torch.full(sh, 0.1, device=self.device)
                t[-1] = 1.0
                return t
            if last == "norm" and ".mix." in name:
                return torch.ones(sh, device=self.device)
            if last in ("ls1", "ls2"):
                return torch.ones(sh, device=self.device)
            if last == "in":               # streams: read their mean, add the
                return torch.full(sh, 1.0 / sh[0], device=self.device)
            if last == "out":              # result to all, keep them apart
                return torch.ones(sh, device=self.device)
            if last == "mix":
                return torch.eye(sh[0], device=self.device)
            if last == "act":              # odd powers, as an activation's
                return torch.tensor([0.5, 0.0, 0.5, 0.0], device=self.device)
            if last == "talk":             # mostly each head's own weights
                return torch.eye(sh[0], device=self.device) + 0.02 * \
                    torch.randn(sh, generator=gen, device=self.device)
            if last in ("norm", "norm1", "norm2", "norm1b", "norm2b"):
                return torch.full(sh, 1.0 - self.norm_off, device=self.device)
            if name.endswith("i.b") or last == "correction":
                return torch.zeros(sh, device=self.device)
            if name.endswith("f.b") or name.endswith("a2.b"):
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

        def norm(t):
            return vec(t.expand(s.hidden) if s.scalar_norms else t,
                       wp).contiguous()

        self.embed = mat(get("embed"))
        self.head = self.embed if s.tied else mat(get("head"))
        self.pos_table = mat(get("pos")) if s.positions else None
        self.embed_norm = norm(get("embed.norm")) if s.embed_norm else None
        self.final_norm = norm(get("final.norm")) + self.norm_off
        # ahead of the head; the logits' scale goes into it
        self.head_norm = self.final_norm * s.logit_scale
        built: dict[int, BlockWeights] = {}
        for i, ly in enumerate(s.layers):
            if ly.weights_of is None:
                built[i] = self._assemble_layer(i, ly, get, mat, norm)
        self.layers = [built[s.owner(i)] for i in range(len(s.layers))]
        self.averages = [get(f"l{i}.dwa").float().contiguous()
                         for i in range(len(s.layers))] \
            if s.depth_average else []

    def _assemble_latent(self, p: str, mx: LatentMixer, get, mat) -> dict:
        h, pd, (kr, r) = mx.heads, head_pad(mx), latent_pad(mx)
        qr, k = pad64(mx.q_rank), mx.kv_rank
        down = mat(get(p + "dkv"))
        wmix = torch.cat([mat(get(p + "dq"), qr), _pad(down[:k], kr,
                                                       down.shape[1]),
                          _pad(down[k:], r, down.shape[1]),
                          mat(get(p + "g"))])
        uq = mat(get(p + "uq")).view(h, mx.dim + mx.rot_dim, qr)
        uk = get(p + "uk").to(self.dtype).view(h, mx.dim, k)
        uv = _pad(get(p + "uv").to(self.dtype).view(h, mx.vdim, k), h, pd, kr)
        uq = torch.cat([_pad(uq[:, :mx.dim], h, pd, qr),
                        _pad(uq[:, mx.dim:], h, r, qr)], dim=1)
        uk = _pad(uk, h, pd, kr)
        return dict(
            wmix=wmix, wuq=uq.reshape(h * (pd + r), qr).contiguous(),
            wuk=uk.transpose(1, 2).contiguous(), wuv=uv.contiguous(),
            wo=_pad_heads(get(p + "o").to(self.dtype).T, h, pd).T,
            wukv=torch.cat([uk, uv], dim=1).contiguous()
            if self.dtype == torch.bfloat16 else None,
            qnorm=_pad(get(p + "dq.norm").float(), qr),
            kvnorm=_pad(get(p + "dkv.norm").float(), kr))

    def _assemble_talk(self, i: int, mx: TalkingMixer, get, mat) -> dict:
        p, h, g, d, pd = f"l{i}.mix.", mx.heads, mx.kv_heads, mx.dim, \
            head_pad(mx)
        order = _pair_order(d, mx.rot_dims).to(self.device)

        def heads(t, n):            # rows [n * d, ...] reordered, padded
            t = t.view(n, d, *t.shape[1:])[:, order]
            return _pad_heads(t.reshape(n * d, *t.shape[2:]), n, pd)

        talk = get(p + "talk").float().contiguous()
        nh = -(-h // 8)             # heads of a wave in the tiled kernel
        if nh <= 4:
            lift = 0
            if talk.abs().max() > 0:
                lift = int(torch.log2(talk.abs().max()).ceil())
            at = torch.tensor([k // nh * 4 + k % nh for k in range(h)],
                              device=self.device)
            talk16 = talk.new_zeros(32, 32)
            talk16[at.unsqueeze(1), at] = talk * 2.0 ** -lift
            talk16 = talk16.half()
        return dict(
            wmix=torch.cat([heads(mat(get(p + "q")), h),
                            heads(mat(get(p + "k")), g)]),
            # a head's columns in the order of its values
            wo=_pad_heads(get(p + "o").to(self.dtype).T.reshape(h, d, -1)
                          [:, order].reshape(h * d, -1), h, pd).T,
            talk=Talk(h, d, mx.scale, mx.cap, mx.chunk, self.rot[i],
                      torch.cat([heads(get(p + "q.b").float(), h),
                                 heads(get(p + "k.b").float(), g)]),
                      _pad(get(p + "q.norm").float()[order], pd),
                      _pad(get(p + "k.norm").float()[order], pd), talk,
                      *((talk16, 2.0 ** (lift - 14)) if nh <= 4 else ())))

    def _assemble_layer(self, i: int, ly, get, mat, norm) -> BlockWeights:
        s, mx, ff, wp = self.spec, ly.mixer, ly.ff, self.width
        p = f"l{s.number(i)}."
        if isinstance(mx, TalkingMixer):
            parts = self._assemble_talk(i, mx, get, mat)
        elif isinstance(mx, LatentMixer):
            parts = self._assemble_latent(p + "mix.", mx, get, mat)
        elif isinstance(mx, ParallelMixer):
            # one row of projections, and one output projection: the parts'
            # scales go into the kernels behind which their outputs are rounded
            parts = self._assemble_rows(p + "mix.left.", mx.left, get, mat)
            right = self._assemble_rows(p + "mix.right.", mx.right, get, mat)
            for name, dim in (("wmix", 0), ("wo", 1)):
                right[name] = torch.cat([parts[name], right[name]], dim=dim)
            right["mnorm"] = right["mnorm"] * mx.right_scale
            parts |= right
        else:
            parts = self._assemble_rows(p + "mix.", mx, get, mat)
        wmix = parts.pop("wmix")
        wmix = _pad(wmix, -(-wmix.shape[0] // 128) * 128, wp).contiguous()
        wo = parts.pop("wo")

        def norms(k):               # behind a sublayer (scaled), ahead of it
            t = norm(get(f"{p}norm{k}b" if s.pre_norms else f"{p}norm{k}"))
            if s.layer_scale:
                t *= _pad(get(f"{p}ls{k}").float(), wp)
            return t, norm(get(f"{p}norm{k}")) if s.pre_norms else None

        def streams(k):             # how a sublayer mixes them, and reads
            if not s.streams:
                return None, None
            t = f"{p}hc{k}."
            return torch.cat([get(t + "mix").float().flatten(),
                              get(t + "out").float()]), \
                get(t + "in").float().contiguous()

        norm1, pre1 = norms(1)
        w = BlockWeights(
            wmix=wmix, wo=_pad(wo, wp, wo.shape[1]).contiguous(),
            norm1=norm1, pre1=pre1, **parts)
        w.hc1, w.read1 = streams(1)
        if ff is None:
            return w
        w.norm2, w.pre2 = norms(2)
        w.hc2, w.read2 = streams(2)
        fp = pad64(ff.ff)
        if isinstance(ff, PolyFF):
            w.up = mat(get(p + "mlp.up"), fp).contiguous()
            w.down = mat(get(p + "mlp.down"), wp)
            w.act = get(p + "mlp.act").float().contiguous()
            return w
        def gated(t, n):
            return torch.cat([mat(get(t + "gate"), n), mat(get(t + "up"), n)])

        if isinstance(ff, DenseFF):
            w.wgateup = gated(p + "mlp.", fp)
            w.down = mat(get(p + "mlp.down"), wp)
            return w
        w.router = mat(get(p + "mlp.router"))
        if ff.shared is not None:
            t = p + "mlp.shared."
            w.wgateup = gated(t, pad64(ff.shared.ff))
            w.sdown = mat(get(t + "down"), wp)
            w.router = torch.cat([w.router, mat(get(t + "sg"))])
        if ff.corrected:
            w.corr = get(p + "mlp.correction").float().contiguous()
        w.up = torch.empty(ff.experts, fp * (2 if ff.gated else 1), wp,
                           dtype=self.dtype, device=self.device)
        w.down = torch.empty(ff.experts, wp, fp, dtype=self.dtype,
                             device=self.device)
        for e in range(ff.experts):
            up = mat(get(f"{p}mlp.e{e}.up"), fp)
            if ff.gated:
                gate = mat(get(f"{p}mlp.e{e}.gate"), fp)
                up = torch.stack([gate.view(-1, 16, wp), up.view(-1, 16, wp)],
                                 dim=1).view(2 * fp, wp)
            w.up[e] = up
            w.down[e] = mat(get(f"{p}mlp.e{e}.down"), wp)
        return w

    def _assemble_rows(self, p: str, mx, get, mat) -> dict:
        """Tensors of a mixer with one row [q | k | v | output gate]."""
        h = mx.heads
        attn = isinstance(mx, AttentionMixer)
        kv = mx.kv_heads if attn else h
        dk = head_pad(mx) if attn else pad64(mx.dim)
        dv = dk if attn else pad64(mx.vdim)
        g = mat(get(p + "g"))
        by_head = attn and mx.gate == "head"
        out = {"wmix": torch.cat([_pad_heads(mat(get(p + "q")), h, dk),
                                  _pad_heads(mat(get(p + "k")), kv, dk),
                                  _pad_heads(mat(get(p + "v")), kv, dv),
                                  g if by_head else _pad_heads(g, h, dv)]),
               # columns follow the padded heads
               "wo": _pad_heads(get(p + "o").to(self.dtype).T, h, dv).T}
        if attn:
            if mx.sink:
                out["sink"] = get(p + "sink").float()
        elif isinstance(mx, LightningMixer):
            d = torch.tensor(mx.decay, dtype=torch.float64)
            out["decay"] = torch.stack([d, d.clamp(min=1e-30).log()]).float() \
                .to(self.device).contiguous()
            out["mnorm"] = _pad_heads(get(p + "norm").float(), h, dv)
        elif isinstance(mx, GlaMixer):
            out["wgates"] = mat(get(p + "a1")).contiguous()
            wa2 = _pad_heads(get(p + "a2").float(), h, dk)
            out["wa2"] = wa2.T.contiguous()
            out["ba2"] = _pad_heads(get(p + "a2.b").float(), h, dk)
            out["mnorm"] = _pad(get(p + "norm").float(), dv).repeat(h)
        else:
            out["wgates"] = torch.cat([mat(get(p + "i")),
                                       mat(get(p + "f"))]).contiguous()
            out["bgates"] = torch.cat([get(p + "i.b"),
                                       get(p + "f.b")]).float()
            out["mnorm"] = _pad_heads(get(p + "norm").float(), h, dv)
        return out

    def unique_layers(self) -> list[BlockWeights]:
        return list({id(w): w for w in self.layers}.values())

    def gemm_shapes(self) -> tuple[list, list]:
        """(n, k) of the decode projections, and of the gate/up ones."""
        plain = {tuple(self.head.shape)}
        gu = set()
        for w in self.unique_layers():
            plain |= {tuple(w.wmix.shape), tuple(w.wo.shape)}
            if w.wuq is not None:
                plain.add(tuple(w.wuq.shape))
            if w.wgateup is not None:
                gu.add(tuple(w.wgateup.shape))
                plain.add(tuple((w.down if w.sdown is None
                                 else w.sdown).shape))
            if w.act is not None:
                plain |= {tuple(w.up.shape), tuple(w.down.shape)}
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
        ts = [self.embed, self.pos_table, self.final_norm, self.embed_norm,
              *self.averages]
        if self.head is not self.embed:
            ts.append(self.head)
        for w in self.unique_layers():
            ts += [t for t in vars(w).values() if not isinstance(t, Talk)]
            if w.talk is not None:
                ts += [w.talk.bias, w.talk.qnorm, w.talk.knorm, w.talk.talk,
                       w.talk.talk16]
        return sum(t.numel() * t.element_size() for t in ts if t is not None)

    # -- layers ------------------------------------------------------------

    def _mix(self, i: int, w: BlockWeights, mx, xb: torch.Tensor,
             st: StepMeta) -> torch.Tensor:
        c, eps = self.cache, self.spec.norm_eps
        rows = _linear(xb, w.wmix)
        if isinstance(mx, ParallelMixer):
            o = torch.empty(xb.shape[0], w.wo.shape[1], dtype=xb.dtype,
                            device=xb.device)
            at = self._attend(i, w, mx.left, rows, st, o, mx.left_scale,
                              mx.right)
            hops.lightning(rows[:, at:], c.S[i], w.decay, w.mnorm, st,
                           mx.right.vdim, eps,
                           o[:, mx.left.heads * c.k[i].shape[3]:])
        elif isinstance(mx, LightningMixer):
            dv, dk = c.S[i].shape[2:]
            hops.silu_cols(rows, 0, mx.heads * (2 * dk + dv))
            o = hops.lightning(rows, c.S[i], w.decay, w.mnorm, st, mx.vdim,
                               eps)
        elif isinstance(mx, AttentionMixer):
            o = torch.empty(xb.shape[0], w.wo.shape[1], dtype=xb.dtype,
                            device=xb.device)
            self._attend(i, w, mx, rows, st, o)
        elif isinstance(mx, LatentMixer):
            cq = hops.latent_rows(rows, c.lat[i], st, self.rot[i], w.qnorm,
                                  w.kvnorm, mx.q_rank, mx.kv_rank, eps)
            at = w.qnorm.shape[0] + c.lat[i].shape[2]
            o = hops.latent_attn(_linear(cq, w.wuq), c.lat[i], st, self.rot[i],
                                 w.wuk, w.wuv, w.wukv, mx.scale,
                                 rows[:, at:at + mx.heads])
        elif isinstance(mx, TalkingMixer):
            q = hops.talk_rows(rows, c.v[i], c.inv[i], st, w.talk, eps)
            o = hops.talk_attn(q, c.v[i], c.inv[i], st,
                               w.talk).view(xb.shape[0], -1)
        elif isinstance(mx, GlaMixer):
            u = hops.proj_f32(xb, w.wgates)
            o = hops.gla(rows, u, w.wa2, w.ba2, c.S[i], w.mnorm, st, mx.dim,
                         mx.vdim, mx.tau, eps)
        else:
            gates = hops.proj_f32(xb, w.wgates, w.bgates)
            o = hops.mlstm(rows, gates, c.S[i], c.m[i], w.mnorm, st, mx.dim,
                           mx.vdim, mx.gate_cap, eps)
        return _linear(o, w.wo)

    def _attend(self, i: int, w: BlockWeights, mx: AttentionMixer,
                rows: torch.Tensor, st: StepMeta, out: torch.Tensor,
                scale: float = 1.0,
                right: Optional[LightningMixer] = None) -> int:
        """Attention of projection rows [q | k | v | gate | ...] into the first
        columns of out, times scale; returns where its part of the rows ends.
        `right` is a recurrence whose part follows: its q, k and v get SiLU."""
        c, h, g = self.cache, mx.heads, mx.kv_heads
        p = c.k[i].shape[3]
        at = (h + 2 * g) * p
        end = at + (h * p if mx.gate == "element" else h)
        silu = (0, 0)
        if right is not None:
            dv, dk = c.S[i].shape[2:]
            silu = (end, right.heads * (2 * dk + dv))
        q = hops.qknorm_kv(rows, c.k[i], c.v[i], st, h, g, mx.dim,
                           self.spec.norm_eps, mx.q_coef, mx.q_every,
                           self.rot[i], silu)
        hops.paged_attn(q, c.k[i], c.v[i], st, mx.scale, w.sink,
                        rows[:, at:end], Keys(mx.window, mx.keep_first),
                        out[:, :h * p], scale)
        return end

    def _gated(self, w: BlockWeights, ff: DenseFF,
               xb: torch.Tensor) -> torch.Tensor:
        if self.gateup_il:
            return _linear_gateup(xb, w.wgateup, _glu(ff))
        return hops.glu(_linear(xb, w.wgateup), _glu(ff))

    def _feed(self, w: BlockWeights, ff, xb: torch.Tensor):
        """Feed-forward output, and, if it is still a row per (token, chosen
        expert), the pairs' weights and those of identity experts; with weighted
        inputs the rows just add up."""
        if isinstance(ff, DenseFF):
            return _linear(self._gated(w, ff, xb), w.down), None, None
        if isinstance(ff, PolyFF):
            z = hops.poly_norm(_linear(xb, w.up), w.act, ff.ff,
                               self.spec.norm_eps)
            return _linear(z, w.down), None, None
        assert isinstance(ff, RoutedFF)
        return hops.moe(xb, hops.proj_f32(xb, w.router), w.up, w.down,
                        self._choice(w, ff))

    @staticmethod
    def _choice(w: BlockWeights, ff: RoutedFF) -> Choice:
        return Choice(ff.top, w.corr, ff.groups, ff.keep,
                      1e-20 if ff.corrected else 0.0, ff.scale, ff.sigmoid,
                      ff.weigh_input, _glu(ff.unit))

    def _run(self, tokens: torch.Tensor, st: StepMeta,
             trail: Optional[list] = None) -> torch.Tensor:
        """The residual stream behind the last layer, f32 [n, W] (or all of
        them, [n, streams, W]); trail collects it (or their sum) behind every
        layer."""
        s = self.spec
        if s.pre_norms:
            return self._run_between_norms(tokens, st, trail)
        if s.streams:
            return self._run_streams(tokens, st, trail)
        n, size, norm = tokens.shape[0], (s.hidden, s.norm_eps), self.norm_off
        hist = None
        if s.depth_average:
            hist = torch.empty(len(s.layers), n, self.width,
                               dtype=torch.float32, device=self.device)
        x, xb = hops.embed(tokens, st.pos, self.embed, self.pos_table,
                           self.embed_norm, norm, *size,
                           out=None if hist is None else hist[0])
        # the stream leaves the embedding's row of hist with the first norm
        xo = x if hist is None else torch.empty_like(x)

        def join(y, g, avg=None, pair_w=None, ident=None):
            """A sublayer's output y joins the stream, by the norm g."""
            nonlocal x, xb
            if s.post_alpha is None:
                hops.post_norm(x, xb, y, g, norm, *size, pair_w)
                return
            if xb is x:
                xb = xo
            hops.sum_norm(x, xo, xb, y, g, norm, s.post_alpha, *size, pair_w,
                          ident, avg)
            x = xo

        for i, (ly, w) in enumerate(zip(s.layers, self.layers)):
            avg = None if hist is None else DepthAverage(
                hist, self.averages[i], i + 1, i + 1 < len(s.layers))
            y = self._mix(i, w, ly.mixer, xb, st)
            join(y, w.norm1, avg if ly.ff is None else None)
            if ly.ff is not None:
                y, pair_w, ident = self._feed(w, ly.ff, xb)
                join(y, w.norm2, avg, pair_w, ident)
            if trail is not None:
                trail.append(x[:, :s.hidden].clone())
        return x

    def _run_between_norms(self, tokens: torch.Tensor, st: StepMeta,
                           trail: Optional[list]) -> torch.Tensor:
        """_run for sublayers between two norms: the norm behind one and the
        norm ahead of the next are one kernel."""
        s = self.spec
        how = (s.norm_groups, s.hidden, s.norm_eps)
        x, _ = hops.embed(tokens, st.pos, self.embed, self.pos_table)
        h = hops.group_norm(x, None, self.layers[0].pre1, *how, self.dtype)
        for i, (ly, w) in enumerate(zip(s.layers, self.layers)):
            ahead = self.layers[i + 1].pre1 if i + 1 < len(s.layers) else None
            y = self._mix(i, w, ly.mixer, h, st)
            h = hops.join_norm(x, y, w.norm1, ahead if ly.ff is None
                               else w.pre2, *how)
            if ly.ff is not None:
                y = self._feed(w, ly.ff, h)[0]
                h = hops.join_norm(x, y, w.norm2, ahead, *how)
            if trail is not None:
                trail.append(x[:, :s.hidden].clone())
        return x

    def _run_streams(self, tokens: torch.Tensor, st: StepMeta,
                     trail: Optional[list]) -> torch.Tensor:
        """_run for several residual streams: taking a sublayer's output in and
        reading the next one's input are one kernel."""
        s, run = self.spec, self.layers
        size = (s.hidden, s.norm_eps)
        x, h = hops.streams_start(tokens, self.embed, s.embed_scale,
                                  run[0].read1, run[0].norm1, *size)
        for i, (ly, w) in enumerate(zip(s.layers, run)):
            ahead = (run[i + 1].read1, run[i + 1].norm1) \
                if i + 1 < len(run) else (None, None)
            y = self._mix(i, w, ly.mixer, h, st)
            h = hops.streams_join(x, y, w.hc1, *(
                ahead if ly.ff is None else (w.read2, w.norm2)), *size)
            if isinstance(ly.ff, RoutedFF):
                y, extra = self._feed_pairs(w, ly.ff, h)
                h = hops.streams_join(x, y, w.hc2, *ahead, *size, ly.ff.top,
                                      extra)
            elif ly.ff is not None:
                h = hops.streams_join(x, self._feed(w, ly.ff, h)[0], w.hc2,
                                      *ahead, *size)
            if trail is not None:
                trail.append(x[..., :s.hidden].sum(1))
        return x

    def _feed_pairs(self, w: BlockWeights, ff: RoutedFF, h: torch.Tensor
                    ) -> tuple[torch.Tensor, Optional[tuple]]:
        """Experts' outputs by (token, chosen expert), which just add up; and
        the shared expert's with the logits of its gate."""
        z = hops.proj_f32(h, w.router)
        y, _, _ = hops.moe(h, z[:, :ff.outputs], w.up, w.down,
                           self._choice(w, ff))
        if ff.shared is None:
            return y, None
        return y, (_linear(self._gated(w, ff.shared, h), w.sdown),
                   z[:, ff.outputs:])

    def _normed(self, x: torch.Tensor, rows: Optional[torch.Tensor],
                w: torch.Tensor) -> torch.Tensor:
        s = self.spec
        if s.streams:
            return hops.streams_norm(x, rows, w, s.hidden, s.norm_eps,
                                     self.dtype)
        if s.norm_groups > 1:
            return hops.group_norm(x, rows, w, s.norm_groups, s.hidden,
                                   s.norm_eps, self.dtype)
        return hops.norm_rows(x, rows, w, 0.0, s.hidden, s.norm_eps,
                              self.dtype)

    def _head(self, x: torch.Tensor, rows: Optional[torch.Tensor]
              ) -> torch.Tensor:
        return _linear(self._normed(x, rows, self.head_norm),
                       self.head).float()

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
        # decode rows, short portions, longer ones
        order = sorted(range(len(entries)), key=lambda i: (
            len(entries[i][1]) > 1) + (len(entries[i][1]) > _ABSORB))
        starts = [int(self.cache.lens[e[0]]) for e in entries]
        self.cache.extend([e[0] for e in entries],
                          [len(e[1]) for e in entries])
        off, first = 0, {}
        toks, pos, slot = [], [], []
        segs, tiles, chunks, csegs = [], [], [], []
        litems, ltiles = [], []
        nd = absorbed = lrows = 0
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
            if ln <= _ABSORB:
                absorbed += ln
            elif self.expands:
                total = p0 + ln            # gathered in blocks of 32 rows
                for c in range(0, total, PAGE):
                    have = min(PAGE, total - c)
                    litems.append((c // PAGE, sl, lrows + c,
                                   have + 256 * (-(-have // 32) * 32)))
                ltiles += [(off, ln, lrows, q0, p0, 0, 0, 0)
                           for q0 in range(0, ln, 128)]
                lrows += -(-total // 32) * 32
            off += ln
        talks = [self._chunk_portions(segs, c) for c in self.chunks]
        ids_np = np.concatenate(toks)
        if ids_np.min() < 0 or ids_np.max() >= self.spec.vocab:
            raise ValueError("token id outside of the vocabulary")
        want = [first[i] + w for i, e in enumerate(entries) for w in e[2]]
        tokens = self.up.upload(ids_np)
        parts = [np.concatenate(pos), np.concatenate(slot), np.asarray(want),
                 np.asarray(segs), np.asarray(tiles), np.asarray(chunks),
                 np.asarray(csegs), np.asarray(litems), np.asarray(ltiles)]
        for t in talks:
            parts += t[2:]
        dev = self._upload_ints(parts)
        mixed = bool(tiles)
        st = StepMeta(nd=nd, pos=dev[0], slot=dev[1], table=self.cache.table,
                      max_len=self.max_seq,
                      segs=dev[3].view(-1, 4) if mixed else None,
                      tiles=dev[4].view(-1, 8) if mixed else None,
                      chunks=dev[5].view(-1, 4) if mixed else None,
                      chunk_segs=dev[6].view(-1, 4) if mixed else None,
                      absorbed=absorbed, lat_rows=lrows,
                      lat_items=dev[7].view(-1, 4) if litems else None,
                      lat_tiles=dev[8].view(-1, 8) if ltiles else None)
        for k, (c, t) in enumerate(zip(self.chunks, talks)):
            if t[0]:
                items, t16, t128 = dev[9 + 3 * k:12 + 3 * k]
                st.talk[c] = ChunkPortions(*t[:2], items.view(-1, 4),
                                           t16.view(-1, 8), t128.view(-1, 8))
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
        h = self._normed(x, None, self.final_norm)
        h = h[:, :self.spec.hidden].float()
        return logits, torch.stack(
            [h[first[i]:first[i] + len(e[1])].mean(0)
             for i, e in enumerate(entries)])

    @staticmethod
    def _chunk_portions(segs: list, chunk: int) -> tuple:
        """The fields of ChunkPortions for the portions among segs, on the
        host."""
        pages, items, tiles = 0, [], {16: [], 128: []}
        for off, ln, sl, p0 in segs:
            if ln <= _ABSORB:
                continue
            page0 = p0 // chunk * chunk // PAGE
            have = np.arange(page0, -(-(p0 + ln) // PAGE))
            items.append(np.stack(
                [have, np.full_like(have, sl), pages + have - page0,
                 np.minimum(PAGE, p0 + ln - have * PAGE)], axis=1))
            for rows, out in tiles.items():
                q0 = np.arange(0, ln, rows)
                t = np.zeros((len(q0), 8), dtype=np.int64)
                t[:, :6] = (off, ln, pages, 0, p0, page0)
                t[:, 3] = q0
                out.append(t)
            pages += len(have)
        if not pages:
            return 0, 0, [], [], []

        def ordered(t):             # blocks start in this order
            span = (t[:, 3] + t[:, 4]) % chunk
            return t[np.argsort(-span, kind="stable")]

        t16, t128 = (ordered(np.concatenate(t)) for t in tiles.values())
        span = int(((t16[:, 3] + t16[:, 4]) % chunk).max()) + 16
        return pages, span, np.concatenate(items), t16, t128

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
                      max_len=self.max_seq, absorbed=tokens.shape[0])
        x = self._run(tokens, st)
        self.cache.seq_lens.index_add_(
            0, slots, torch.ones_like(slot_map))
        return self._head(x, None)
