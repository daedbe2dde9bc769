"""ctypes binding to libgridllm_hybrid.so, libgridllm_latent.so and
libgridllm_talk.so: the gfx950 kernels of the layer-list models
(csrc/gridllm_hybrid.hip, _latent.hip and _talk.hip). Same contract as hip_ops:
launches go onto torch's current stream, a missing library raises, shapes are
checked on the host before a launch.

Every function here has a CPU counterpart of the same signature in
reference_hybrid; ops.hybrid picks one by device.
"""

from __future__ import annotations

import ctypes
import os
from typing import Callable, Optional, Union

import torch
import torch.nn.functional as F

from gridllm_amd.ops.build import lib_path
from gridllm_amd.ops.hip_ops import (HipExtensionMissing, _check,
                                     _check_range)
from gridllm_amd.ops.reference import Glu
from gridllm_amd.ops.reference_hybrid import (ALL_KEYS, Choice, Keys, StepMeta,
                                              Talk)

_libs: dict[str, ctypes.CDLL] = {}
PAGE = 64
_MLSTM, _CHANNELS, _CONSTANT = 0, 1, 2      # kinds of recurrence
LOG2E = 1.4426950408889634

# argument kinds of each entry point after the stream: p pointer, i int,
# l long, f float
_SIGS = {
    "gh_embed": "ipppppppfiiifii",
    "gh_post_norm": "ippppipfiiif",
    "gh_sum_norm": "ipppppippffppiiiiif",
    "gh_norm_rows": "ippppfiiif",
    "gh_group_norm": "ippppppiiiif",
    "gh_poly_norm": "ipppiiif",
    "gh_glu_f32": "ppliffff",
    "gh_proj_f32": "ppppiii",
    "gh_streams_start": "ippppfppiiiifi",
    "gh_streams_join": "iipppippipppiiiif",
    "gh_streams_norm": "ippppiiiif",
    "gh_qknorm_kv": "ipppppippiiiiiiffippiiii",
    "gh_paged_decode": "pppppipppiiiiifiippiifi",
    "gh_paged_prefill": "pppppipiiiifiippiifi",
    "gh_attn_rows_f32": "pppppippiiiifiippiifi",
    "gh_rec_step": "iippppppppiiiiiffi",
    "gh_rec_row_out": "ippppiiiiiif",
    "gh_rec_out": "iipppppppppiiiiiiiiff",
    "gh_mlstm_chunks": "ipppppppppiiiiiiff",
    "gh_gla_decay": "pppppiiiif",
    "gh_gla_chunks": "pppppppiiiiiif",
    "gh_moe_route": "pppppppippiiiiiiffiii",
    "gh_moe_gemm": "iipppppiiiiiffffp",
    "gn_latent_rows": "ippppippppppiiiiiiiif",
    "gn_head_gemm": "ippppiiiiili",
    "gn_latent_decode": "pppppipppppiiiiiiif",
    "gn_latent_attn_f32": "pppppippppiiiiiif",
    "gn_latent_gather": "pppipii",
    "gn_latent_prefill": "ppppipippiiiifpi",
    "gt_talk_rows": "ipppppippppppiiiiiiiif",
    "gt_talk_decode": "pppppippppppp" + "iiiiiiiifff",
    "gt_talk_gather": "pppppipppipiiii",
    "gt_talk_lse": "ppppiiiiifff",
    "gt_talk_prefill": "pppppppiiiiiffffpiii",
    "gt_talk_plain": "ipppppipppppp" + "iiiiiiiff",
}
_LIB_OF = {"gh": "hybrid", "gn": "latent", "gt": "talk"}
_KINDS = {"p": ctypes.c_void_p, "i": ctypes.c_int, "l": ctypes.c_long,
          "f": ctypes.c_float}


def _load(which: str) -> ctypes.CDLL:
    if which not in _libs:
        path = lib_path(_LIB_OF[which])
        if not os.path.exists(path):
            raise HipExtensionMissing(
                f"GridLLM HIP kernel library not found at {path}. Build it "
                "with: python -m gridllm_amd.ops.build (this is required on "
                "GPU machines; there is no eager fallback).")
        lib = ctypes.CDLL(path)
        for name, sig in _SIGS.items():
            if not name.startswith(which):
                continue
            fn = getattr(lib, name)
            fn.argtypes = [ctypes.c_void_p] + [_KINDS[c] for c in sig]
            fn.restype = ctypes.c_int
        _libs[which] = lib
    return _libs[which]


_fns: dict[str, Callable] = {}


def _call(name: str, *args) -> None:
    """Launch by entry point. A prompt step is a hundred and more of these, so
    tensors become plain addresses (which the signature converts)."""
    fn = _fns.get(name)
    if fn is None:
        fn = _fns[name] = getattr(_load(name[:2]), name)
    stream = torch._C._cuda_getCurrentRawStream(torch.cuda.current_device())
    rc = fn(stream, *[a.data_ptr() if isinstance(a, torch.Tensor) else a
                      for a in args])
    if rc:
        _check(rc, name)


def _f32(t: torch.Tensor) -> int:
    if t.dtype == torch.float32:
        return 1
    if t.dtype == torch.bfloat16:
        return 0
    raise TypeError(f"layer-list kernels run in bf16 or fp32, not {t.dtype}")


def _dense(*ts: Optional[torch.Tensor]) -> None:
    for t in ts:
        if t is not None and not t.is_contiguous():
            raise ValueError("kernel operand is not contiguous")


def embed(tok: torch.Tensor, pos: torch.Tensor, emb: torch.Tensor,
          ptab: Optional[torch.Tensor], w: Optional[torch.Tensor] = None,
          w_off: float = 0.0, width: int = 0, eps: float = 0.0,
          out: Optional[torch.Tensor] = None
          ) -> tuple[torch.Tensor, torch.Tensor]:
    """f32 residual embed[tok], plus ptab[pos] if there is a table, normed if
    there are norm weights w; and its copy in the weights' type (the same
    tensor if that is f32). `out` takes the residual."""
    n, wp = tok.shape[0], emb.shape[1]
    _dense(tok, pos, emb, ptab, w, out)
    x = torch.empty(n, wp, dtype=torch.float32, device=tok.device) \
        if out is None else out
    assert x.shape == (n, wp)
    f = _f32(emb)
    xb = x if f else torch.empty(n, wp, dtype=emb.dtype, device=tok.device)
    _call("gh_embed", f, x, None if f else xb, emb, ptab, tok, pos, w, w_off,
          n, wp, width, eps, emb.shape[0], 0 if ptab is None else ptab.shape[0])
    return x, xb


def post_norm(x: torch.Tensor, xb: torch.Tensor, y: torch.Tensor,
              w: torch.Tensor, w_off: float, width: int, eps: float,
              pair_w: Optional[torch.Tensor] = None) -> None:
    """x += norm(y), in place, and xb = x in its type. With pair_w [n, top],
    y [n * top, W] is first summed over a token's pairs by these weights."""
    n, wp = x.shape
    top = 0 if pair_w is None else pair_w.shape[1]
    _dense(x, xb, y, w, pair_w)
    assert y.shape == (n * max(1, top), wp) and w.shape == (wp,)
    f = _f32(y)
    _call("gh_post_norm", f, x, None if xb is x else xb, y, pair_w, top, w,
          w_off, n, wp, width, eps)


def sum_norm(x: torch.Tensor, xo: torch.Tensor, xb: torch.Tensor,
             y: torch.Tensor, w: torch.Tensor, w_off: float, alpha: float,
             width: int, eps: float, pair_w: Optional[torch.Tensor] = None,
             ident: Optional[torch.Tensor] = None, avg=None) -> None:
    """xo = norm(alpha x + y), and xb = xo in its type; x may be xo. pair_w as
    in post_norm; ident [n]: weight with which y also holds x itself. With a
    DepthAverage the norm is the layer's result and xo the average."""
    n, wp = x.shape
    top = 0 if pair_w is None else pair_w.shape[1]
    _dense(x, xo, xb, y, w, pair_w, ident)
    assert y.shape == (n * max(1, top), wp) and w.shape == (wp,)
    assert xo.shape == x.shape and (ident is None or ident.shape == (n,))
    hist = coef = None
    at = keep = 0
    if avg is not None:
        hist, coef, at, keep = avg.hist, avg.coef, avg.at, int(avg.store)
        _dense(hist, coef)
        assert hist.shape[1:] == (n, wp) and 0 < at < coef.shape[0] + 1
        assert coef.shape[0] == at + 1 and hist.shape[0] >= at + keep
    f = _f32(y)
    _call("gh_sum_norm", f, xo, None if xb is xo else xb, x, y, pair_w, top,
          ident, w, w_off, alpha, hist, coef, at, keep, n, wp, width, eps)


def norm_rows(x: torch.Tensor, rows: Optional[torch.Tensor], w: torch.Tensor,
              w_off: float, width: int, eps: float,
              dtype: torch.dtype) -> torch.Tensor:
    """norm(x[rows]) in dtype; rows int32, None for all."""
    m = x.shape[0] if rows is None else rows.shape[0]
    _dense(x, rows, w)
    if rows is not None:
        _check_range("norm_rows.rows", rows, x.shape[0])
    out = torch.empty(m, x.shape[1], dtype=dtype, device=x.device)
    _call("gh_norm_rows", _f32(out), out, x, rows, w, w_off, m, x.shape[1],
          width, eps)
    return out


def group_norm(x: torch.Tensor, rows: Optional[torch.Tensor], w: torch.Tensor,
               groups: int, width: int, eps: float,
               dtype: torch.dtype) -> torch.Tensor:
    """norm(x[rows]) * w in dtype, each of `groups` equal parts of the first
    `width` columns by its own mean; rows int32, None for all."""
    m = x.shape[0] if rows is None else rows.shape[0]
    _dense(x, rows, w)
    assert w.shape == (x.shape[1],) and width % groups == 0
    if rows is not None:
        _check_range("group_norm.rows", rows, x.shape[0])
    out = torch.empty(m, x.shape[1], dtype=dtype, device=x.device)
    _call("gh_group_norm", _f32(out), out, x, None, rows, None, w, m,
          x.shape[1], groups, width // groups, eps)
    return out


def join_norm(x: torch.Tensor, y: torch.Tensor, wy: torch.Tensor,
              w: Optional[torch.Tensor], groups: int, width: int,
              eps: float) -> Optional[torch.Tensor]:
    """x += norm(y) * wy, in place; then norm(x) * w in y's type, if there is a
    w. Norms as in group_norm."""
    n, wp = x.shape
    _dense(x, y, wy, w)
    assert y.shape == x.shape and wy.shape == (wp,) and width % groups == 0
    out = None if w is None else torch.empty_like(y)
    _call("gh_group_norm", _f32(y), out, x, y, None, wy, w, n, wp, groups,
          width // groups, eps)
    return out


def poly_norm(z: torch.Tensor, coef: torch.Tensor, ff: int,
              eps: float) -> torch.Tensor:
    """c0 N(z) + c1 N(z^2) + c2 N(z^3) + c3, N dividing a row by its root mean
    square over the first ff columns (the others are zero); coef f32 [4]."""
    _dense(z, coef)
    assert coef.shape == (4,) and 0 < ff <= z.shape[1]
    out = torch.empty_like(z)
    _call("gh_poly_norm", _f32(z), out, z, coef, z.shape[0], z.shape[1], ff,
          eps)
    return out


def glu_f32(gu: torch.Tensor, glu: Glu) -> torch.Tensor:
    n, f = gu.shape[0], gu.shape[1] // 2
    _dense(gu)
    out = torch.empty(n, f, dtype=torch.float32, device=gu.device)
    _call("gh_glu_f32", out, gu, n, f, *glu)
    return out


def proj_f32(x: torch.Tensor, w: torch.Tensor,
             bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """x @ w.T + bias with an f32 result, for few outputs (router logits,
    gates of a recurrence)."""
    if _f32(x):
        return F.linear(x, w, bias)
    _dense(x, w, bias)
    out = torch.empty(x.shape[0], w.shape[0], dtype=torch.float32,
                      device=x.device)
    _call("gh_proj_f32", out, x, w, bias, x.shape[0], w.shape[0], x.shape[1])
    return out


def streams_start(tok: torch.Tensor, emb: torch.Tensor, scale: float,
                  read: torch.Tensor, w: torch.Tensor, width: int,
                  eps: float) -> tuple[torch.Tensor, torch.Tensor]:
    """Residual streams f32 [n, streams, W], all embed[tok] * scale, and
    norm(sum_s read[s] x_s) * w in the weights' type. read: f32 [streams]."""
    n, (vocab, wp), ns = tok.shape[0], emb.shape, read.shape[0]
    _dense(tok, emb, read, w)
    assert w.shape == (wp,) and tok.dtype == torch.int64
    x = torch.empty(n, ns, wp, dtype=torch.float32, device=tok.device)
    h = torch.empty(n, wp, dtype=emb.dtype, device=tok.device)
    _call("gh_streams_start", _f32(emb), x, h, emb, tok, scale, read, w, n, ns,
          wp, width, eps, vocab)
    return x, h


def streams_join(x: torch.Tensor, y: torch.Tensor, hc: torch.Tensor,
                 read: Optional[torch.Tensor], w: Optional[torch.Tensor],
                 width: int, eps: float, top: int = 0,
                 extra: Optional[tuple] = None) -> Optional[torch.Tensor]:
    """x_t <- sum_s mix[s, t] x_s + put[t] y, in place; then norm(sum_s read[s]
    x_s) * w in y's type, if there is a w. hc f32: mix, then put. With top, y
    [n * top, W] is first summed over a token's pairs; extra (rows [n, W], z f32
    [n, 1], a column view is fine) adds rows times sigmoid(z)."""
    n, ns, wp = x.shape
    _dense(x, y, hc, read, w)
    assert y.shape == (n * max(1, top), wp) and hc.shape == (ns * ns + ns,)
    assert w is None or w.shape == (wp,) and read.shape == (ns,)
    rows = z = None
    if extra is not None:
        rows, z = extra
        _dense(rows)
        assert top and rows.shape == (n, wp) and rows.dtype == y.dtype
        assert z.shape == (n, 1) and z.dtype == torch.float32
    h = None if w is None else torch.empty(n, wp, dtype=y.dtype,
                                           device=y.device)
    _call("gh_streams_join", _f32(y), int(top > 0), x, h, y, top, rows, z,
          0 if z is None else z.stride(0), hc, read, w, n, ns, wp, width, eps)
    return h


def streams_norm(x: torch.Tensor, rows: Optional[torch.Tensor],
                 w: torch.Tensor, width: int, eps: float,
                 dtype: torch.dtype) -> torch.Tensor:
    """norm of the streams' sum at x[rows], times w, in dtype; rows int32, None
    for all."""
    n, ns, wp = x.shape
    m = n if rows is None else rows.shape[0]
    _dense(x, rows, w)
    assert w.shape == (wp,)
    if rows is not None:
        _check_range("streams_norm.rows", rows, n)
    out = torch.empty(m, wp, dtype=dtype, device=x.device)
    _call("gh_streams_norm", _f32(out), out, x, rows, w, m, ns, wp, width, eps)
    return out


def qknorm_kv(qkv: torch.Tensor, kc: torch.Tensor, vc: torch.Tensor,
              st: StepMeta, heads: int, kv_heads: int, dim: int, eps: float,
              coef: float, every: int, rot: Optional[tuple] = None,
              silu: tuple[int, int] = (0, 0)) -> torch.Tensor:
    """Unit-RMS q (with temperature) -> [n, heads, P]; unit-RMS k and v go to
    the pages of kc / vc [pages, kv_heads, 64, P]. rot: cos and sin tables
    [positions, R / 2] by which the first R coordinates of q and k turn first.
    silu: first column and number of columns of qkv that get SiLU in place."""
    n, p = qkv.shape[0], kc.shape[3]
    _dense(qkv, kc, vc, st.table, *(rot or ()))
    assert qkv.shape[1] >= (heads + 2 * kv_heads) * p
    assert sum(silu) <= qkv.shape[1]
    assert rot is None or rot[0].shape == rot[1].shape
    _check_range("qknorm_kv.slot", st.slot, st.table.shape[0])
    q = torch.empty(n, heads, p, dtype=qkv.dtype, device=qkv.device)
    tables = (None, None, 0, 0) if rot is None else \
        (*rot, rot[0].shape[1], rot[0].shape[0])
    _call("gh_qknorm_kv", _f32(qkv), qkv, q, kc, vc, st.table,
          st.table.shape[1], st.pos, st.slot, n, heads, kv_heads, p,
          qkv.shape[1], dim, eps, coef, every, *tables, *silu)
    return q


def silu_cols(rows: torch.Tensor, at: int, count: int) -> None:
    """SiLU on `count` columns of rows from `at` on, in place."""
    n, ld = rows.shape
    _dense(rows)
    assert 0 <= at and 0 < count <= ld - at
    _call("gh_qknorm_kv", _f32(rows), rows, None, None, None, None, 0, None,
          None, n, 0, 0, 64, ld, 1, 0.0, 0.0, 1, None, None, 0, 0, at, count)


def paged_attn(q: torch.Tensor, kc: torch.Tensor, vc: torch.Tensor,
               st: StepMeta, scale: float, sink: Optional[torch.Tensor],
               gate: Optional[torch.Tensor], keys: Keys = ALL_KEYS,
               out: Optional[torch.Tensor] = None,
               oscale: float = 1.0) -> torch.Tensor:
    """Causal attention of a step's tokens over their sequences' pages.
    q [n, heads, P]; sink [heads] f32; gate [n, heads], or [n, heads * P] for a
    gate per element (a column view of the projection rows is fine). `out`
    takes the result [n, heads * P], a column view too; oscale multiplies it.
    Without it the result is [n, heads, P]."""
    n, h, p = q.shape
    if out is None:
        out = torch.empty_like(q)
        paged_attn(q, kc, vc, st, scale, sink, gate, keys,
                   out.view(n, h * p), oscale)
        return out
    g = kc.shape[1]
    _dense(q, kc, vc, st.table, sink)
    assert out.shape == (n, h * p) and out.stride(1) == 1
    ld = el = 0
    if gate is not None:
        assert gate.stride(1) == 1 and gate.dtype == q.dtype
        assert gate.shape in ((n, h), (n, h * p))
        ld, el = gate.stride(0), int(gate.shape[1] != h)
    how = (scale, keys.window, keys.keep, sink, gate, ld, el, oscale,
           out.stride(0))
    per = st.table.shape[1]
    if _f32(q):
        _call("gh_attn_rows_f32", out, q, kc, vc, st.table, per, st.pos,
              st.slot, n, h, g, p, *how)
        return out
    if st.nd:
        groups = h // max(d for d in range(1, 9) if (h // g) % d == 0)
        nsplit = max(1, min(512 // max(1, st.nd * groups),
                            (keys.most(st.max_len) + 255) // 256, 32))
        ws = torch.empty(st.nd * h * nsplit * (p + 2), dtype=torch.float32,
                         device=q.device) if nsplit > 1 else None
        _call("gh_paged_decode", out, q, kc, vc, st.table, per, st.pos,
              st.slot, ws, st.nd, h, g, p, nsplit, *how)
    if st.tiles is not None:
        _call("gh_paged_prefill", out, q, kc, vc, st.table, per, st.tiles,
              st.tiles.shape[0], h, g, p, *how)
    return out


def mlstm(qkv: torch.Tensor, gates: torch.Tensor, S: torch.Tensor,
          m: torch.Tensor, norm: torch.Tensor, st: StepMeta, dim: int,
          vdim: int, cap: float, eps: float) -> torch.Tensor:
    """mLSTM over a step's tokens. qkv rows [H*DK q | H*DK k | H*DV v | H*DV
    output gate | ...]; gates f32 [n, 2 H]; S f32 [slots, H, DV + 1, DK] and
    m f32 [slots, H] are advanced in place. -> [n, H * DV]."""
    n, ld = qkv.shape
    h, dv, dk = S.shape[1], S.shape[2] - 1, S.shape[3]
    _dense(qkv, gates, S, m, norm)
    assert ld >= h * (2 * dk + 2 * dv) and gates.shape == (n, 2 * h)
    f = _f32(qkv)
    qscale = dim ** -0.5
    o = torch.empty(n, h, dv + 4, dtype=torch.float32, device=qkv.device)
    segs, nseg = (st.segs, st.segs.shape[0]) if f and st.segs is not None \
        else (None, st.nd)
    if nseg:
        # rows of the state per block: more for large batches, where the grid
        # is full anyway and a block amortises its loads of q and k
        rpb = 128 if nseg * h * (dv + 1) >= 128 * 2048 else 32
        _call("gh_rec_step", f, _MLSTM, o, S, m, qkv, gates, segs, st.pos,
              st.slot, nseg, h, dk, dv, ld, qscale, cap, rpb)
    nplain = 0
    if not f and st.chunks is not None:
        nplain = n - st.nd
        nch = st.chunks.shape[0]
        ds = torch.empty(nch, h, dv + 1, dk, dtype=torch.float32,
                         device=qkv.device)
        scal = torch.empty(nch, h, 4, dtype=torch.float32, device=qkv.device)
        _call("gh_mlstm_chunks", 0, o, S, m, ds, scal, qkv, gates, st.chunks,
              st.chunk_segs, nch, st.chunk_segs.shape[0], h, dk, dv, ld,
              qscale, cap)
    out = torch.empty(n, h * dv, dtype=qkv.dtype, device=qkv.device)
    _call("gh_rec_out", f, 0, out, o, m, qkv, gates, segs, st.pos, st.slot,
          norm, nseg, st.nd, nplain, h, dk, dv, ld, vdim, cap, eps)
    return out


def lightning(rows: torch.Tensor, S: torch.Tensor, decay: torch.Tensor,
              norm: torch.Tensor, st: StepMeta, vdim: int, eps: float,
              out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Lightning attention over a step's tokens. rows [H*DK q | H*DK k | H*DV v
    | H*DV gate | ...] with SiLU on q, k and v already (a column view is fine);
    decay f32 [2, H]: the decays and their logarithms; S f32 [slots, H, DV, DK]
    is advanced in place. -> [n, H * DV], in `out` if given."""
    n, ld = rows.shape[0], rows.stride(0)
    h, dv, dk = S.shape[1:]
    _dense(S, decay, norm)
    assert rows.stride(1) == 1 and rows.shape[1] >= h * (2 * dk + 2 * dv)
    assert decay.shape == (2, h) and norm.shape == (h * dv,)
    f, dev = _f32(rows), rows.device
    if out is None:
        out = torch.empty(n, h * dv, dtype=rows.dtype, device=dev)
    assert out.shape == (n, h * dv) and out.stride(1) == 1
    o = torch.empty(n, h, dv + 4, dtype=torch.float32, device=dev)
    # the exact mode walks every portion token by token
    segs, nseg = (st.segs, st.segs.shape[0]) if f and st.segs is not None \
        else (None, st.nd)
    if nseg:
        rpb = 128 if nseg * h * dv >= 128 * 2048 else 32
        _call("gh_rec_step", f, _CONSTANT, o, S, None, rows, decay[0], segs,
              st.pos, st.slot, nseg, h, dk, dv, ld, 1.0, 0.0, rpb)
    if not f and st.chunks is not None:
        nch = st.chunks.shape[0]
        ds = torch.empty(nch, h, dv, dk, dtype=torch.float32, device=dev)
        scal = torch.empty(nch, h, 4, dtype=torch.float32, device=dev)
        _call("gh_mlstm_chunks", 1, o, S, None, ds, scal, rows, decay[1],
              st.chunks, st.chunk_segs, nch, st.chunk_segs.shape[0], h, dk, dv,
              ld, 1.0, 0.0)
    at = h * (2 * dk + dv)
    _call("gh_rec_row_out", f, out, o, rows[:, at:], norm, n, h, dv, ld,
          out.stride(0), h * vdim, eps)
    return out


# up to this many (token, expert) pairs, mostly of different experts, the
# 16-row kernel fills the chip better than 128 x 128 tiles do
_FEW_PAIRS = 64


def moe(x: torch.Tensor, logits: torch.Tensor, up: torch.Tensor,
        down: torch.Tensor, how: Union[int, Choice]
        ) -> tuple[torch.Tensor, torch.Tensor, Optional[torch.Tensor]]:
    """Routed experts. x [n, W]; logits f32 [n, E + identities] (a column view
    is fine); down [E, W, F]; up [E, F, W] with squared ReLU, or [E, 2 F, W] in
    turns of 16 gate | 16 up rows for the gated unit how.glu. Returns the chosen
    experts' outputs [n * top, W] in pair order, their weights f32 [n, top]
    (zero, and the row undefined, where the choice is an identity) and the
    identities' summed weights [n]."""
    if isinstance(how, int):
        how = Choice(how)
    n, w = x.shape
    e, rows, ff = up.shape[0], up.shape[1], down.shape[2]
    outs, top = logits.shape[1], how.top
    _dense(x, up, down, how.corr)
    assert logits.stride(1) == 1 and logits.dtype == torch.float32
    assert not (how.sigmoid and (how.corr is not None or outs > e))
    assert rows in (ff, 2 * ff) and up.shape[2] == w == down.shape[1]
    assert outs >= e and (how.corr is None or how.corr.shape == (outs,))
    dev, f = x.device, _f32(x)
    pairs = n * top
    bm = 16 if f or pairs <= _FEW_PAIRS else 128
    max_tiles = min(pairs, e + pairs // bm)
    ints = torch.empty(3 * pairs, dtype=torch.int32, device=dev)
    idx, rank, order = ints[:pairs], ints[pairs:2 * pairs], ints[2 * pairs:]
    counts = torch.zeros(outs, dtype=torch.int32, device=dev)
    tiles = torch.empty(max_tiles + 1, 4, dtype=torch.int32, device=dev)
    wt = torch.empty(n, top, dtype=torch.float32, device=dev)
    ident = torch.empty(n, dtype=torch.float32, device=dev) \
        if outs > e else None
    _call("gh_moe_route", idx, wt, rank, counts, order, tiles, logits,
          logits.stride(0), how.corr, ident, n, outs, e, top, how.groups,
          how.keep, how.eps, how.scale, int(how.sigmoid), bm, max_tiles)
    act = torch.empty(pairs, ff, dtype=x.dtype, device=dev)
    _call("gh_moe_gemm", f, rows // ff, act, x, up, tiles, order, top, rows, w,
          bm, max_tiles, *how.glu, wt if how.weigh_input else None)
    ye = torch.empty(pairs, w, dtype=x.dtype, device=dev)
    _call("gh_moe_gemm", f, 0, ye, act, down, tiles, order, top, w, ff, bm,
          max_tiles, *how.glu, None)
    return ye, wt, ident


def latent_rows(rows: torch.Tensor, lat: torch.Tensor, st: StepMeta,
                rot: tuple, qnorm: torch.Tensor, kvnorm: torch.Tensor,
                qtrue: int, ktrue: int, eps: float) -> torch.Tensor:
    """From projection rows [q latent | latent | rotated part | ...]: the normed
    query latents [n, QR]; normed latent and rotated part go to the pages of
    lat [pages, 64, KR + R]. rot: cos and sin tables [positions, R / 2]."""
    n, ld = rows.shape
    qr, kr = qnorm.shape[0], kvnorm.shape[0]
    r = lat.shape[2] - kr
    _dense(rows, lat, st.table, qnorm, kvnorm, *rot)
    assert ld >= qr + kr + r and rot[0].shape == rot[1].shape
    assert rot[0].shape[1] == r // 2
    _check_range("latent_rows.slot", st.slot, st.table.shape[0])
    cq = torch.empty(n, qr, dtype=rows.dtype, device=rows.device)
    _call("gn_latent_rows", _f32(rows), rows, cq, lat, st.table,
          st.table.shape[1], st.pos, st.slot, qnorm, kvnorm, *rot,
          rot[0].shape[0], n, qr, qtrue, kr, ktrue, r, ld, eps)
    return cq


def _head_gemm(out, x, w, gate, rows, hx):
    """out[:rows] = per-head x w^T; w [H, N, K]; hx: stride of x's heads."""
    h, nn, k = w.shape
    _dense(w)
    assert x.stride(-1) == 1 and x.dtype == w.dtype == out.dtype
    _call("gn_head_gemm", _f32(x), out, x, w, gate,
          0 if gate is None else gate.stride(0), rows, h, nn, k, x.stride(0),
          hx)


def latent_attn(q: torch.Tensor, lat: torch.Tensor, st: StepMeta, rot: tuple,
                wuk: torch.Tensor, wuv: torch.Tensor,
                wukv: Optional[torch.Tensor], scale: float,
                gate: torch.Tensor) -> torch.Tensor:
    """Latent attention of a step's tokens. q rows [H, P + R], the last R yet to
    be rotated; wuk [H, KR, P], wuv [H, P, KR], wukv [H, 2 P, KR] (keys, then
    values; bf16 only); gate [n, >= H], a column view is fine. -> [n, H * P]"""
    h, kr, p = wuk.shape
    n, r, per = q.shape[0], lat.shape[2] - kr, st.table.shape[1]
    _dense(q, lat, st.table, *rot)
    assert q.shape[1] == h * (p + r) and wuv.shape == (h, p, kr)
    assert gate.stride(1) == 1 and gate.dtype == q.dtype
    f, nrot = _f32(q), rot[0].shape[0]
    out = torch.empty(n, h * p, dtype=q.dtype, device=q.device)
    na = n if f else st.absorbed
    if na:
        ql = torch.empty(na, h, kr, dtype=q.dtype, device=q.device)
        _head_gemm(ql, q, wuk, None, na, p + r)
        ol = torch.empty_like(ql)
        if f:
            _call("gn_latent_attn_f32", ol, ql, q, lat, st.table, per, st.pos,
                  st.slot, *rot, nrot, na, h, p, kr, r, scale)
        else:
            # a CU takes one block of 32 heads, or two of 16
            blocks, fill = (na * -(-h // 32), 256) if h > 16 else (na, 512)
            nsplit = max(1, min(fill // blocks, -(-st.max_len // 128), 32))
            ws = torch.empty(na * h * nsplit * (kr + 2), dtype=torch.float32,
                             device=q.device) if nsplit > 1 else None
            _call("gn_latent_decode", ol, ql, q, lat, st.table, per, st.pos,
                  st.slot, ws, *rot, nrot, na, h, p, kr, r, nsplit, scale)
        _head_gemm(out, ol.view(na, h * kr), wuv, gate, na, kr)
    if na < n:
        rows = torch.empty(st.lat_rows, kr + r, dtype=q.dtype,
                           device=q.device)
        _call("gn_latent_gather", rows, lat, st.table, per, st.lat_items,
              st.lat_items.shape[0], kr + r)
        e = F.linear(rows[:, :kr], wukv.view(h * 2 * p, kr))
        _call("gn_latent_prefill", out, q, e, rows, kr + r, st.lat_tiles,
              st.lat_tiles.shape[0], *rot, nrot, h, p, r, scale, gate,
              gate.stride(0))
    return out


def gla(rows: torch.Tensor, u: torch.Tensor, wa2: torch.Tensor,
        ba2: torch.Tensor, S: torch.Tensor, norm: torch.Tensor, st: StepMeta,
        dim: int, vdim: int, tau: float, eps: float) -> torch.Tensor:
    """Gated linear attention over a step's tokens. rows [H*DK q | H*DK k |
    H*DV v | H*DV gate | ...]; u f32 [n, rank], wa2 f32 [rank, H*DK] and ba2
    give the decays' logits; S f32 [slots, H, DV, DK] is advanced in place.
    -> [n, H * DV]."""
    n, ld = rows.shape
    h, dv, dk = S.shape[1:]
    _dense(rows, u, wa2, ba2, S, norm)
    assert ld >= h * (2 * dk + 2 * dv) and u.shape == (n, wa2.shape[0])
    assert wa2.shape[1] == ba2.shape[0] == h * dk and norm.shape == (h * dv,)
    f, dev = _f32(rows), rows.device
    qscale = dim ** -0.5
    # the exact mode walks every portion token by token
    nch = 0 if f or st.chunks is None else st.chunks.shape[0]
    b = torch.empty(n, h * dk, dtype=torch.float32, device=dev)
    _call("gh_gla_decay", b, u, wa2, ba2, st.chunks if nch else None,
          st.nd if nch else n, nch, wa2.shape[0], h * dk, 1.0 / tau)
    o = torch.empty(n, h, dv + 4, dtype=torch.float32, device=dev)
    segs, nseg = (st.segs, st.segs.shape[0]) if f and st.segs is not None \
        else (None, st.nd)
    if nseg:
        rpb = 128 if nseg * h * dv >= 128 * 2048 else 32
        _call("gh_rec_step", f, _CHANNELS, o, S, None, rows, b, segs, st.pos,
              st.slot, nseg, h, dk, dv, ld, qscale, 0.0, rpb)
    if nch:
        ds = torch.empty(nch, h, dv, dk, dtype=torch.float32, device=dev)
        _call("gh_gla_chunks", o, S, ds, rows, b, st.chunks, st.chunk_segs,
              nch, st.chunk_segs.shape[0], h, dk, dv, ld, qscale)
    out = torch.empty(n, h * dv, dtype=rows.dtype, device=dev)
    _call("gh_rec_out", f, 1, out, o, None, rows, None, None, st.pos, st.slot,
          norm, 0, 0, n, h, dk, dv, ld, vdim, 0.0, eps)
    return out


def talk_rows(rows: torch.Tensor, vc: torch.Tensor, inv: torch.Tensor,
              st: StepMeta, tk: Talk, eps: float) -> torch.Tensor:
    """From projection rows [q H*P | k G*P | ...] without their bias: normed and
    rotated queries [n, H, P]; k goes to the pages of vc [pages, G, 64, P], and
    1 / rms(k) to inv f32 [pages, G, 64]."""
    n, ld = rows.shape
    h, (g, _, p) = tk.heads, vc.shape[1:]
    _dense(rows, vc, inv, st.table, tk.bias, tk.qnorm, *tk.rot)
    assert ld >= (h + g) * p and tk.bias.shape == ((h + g) * p,)
    assert inv.shape == vc.shape[:3] and tk.qnorm.shape == (p,)
    _check_range("talk_rows.slot", st.slot, st.table.shape[0])
    q = torch.empty(n, h, p, dtype=rows.dtype, device=rows.device)
    _call("gt_talk_rows", _f32(rows), rows, q, vc, inv, st.table,
          st.table.shape[1], st.pos, st.slot, tk.bias, tk.qnorm, *tk.rot,
          tk.rot[0].shape[0], n, h, g, p, 2 * tk.rot[0].shape[1], ld, tk.dim,
          eps)
    return q


def _talk_sizes(tk: Talk, g: int, p: int) -> tuple[bool, bool]:
    """Whether the one-pass and the tiled kernels take these sizes."""
    h, nh = tk.heads, -(-tk.heads // 8)
    one = h <= 64 and g * p <= 1024 and not (p == 256 and g > 2 and h > 32) \
        and tk.cap <= 128
    return one, one and nh <= 4 and nh * p <= 512


def _talk_splits(rows: int, heads: int, seen: int) -> int:
    """Into how many parts a decode row's keys are split. (A part's sums are as
    large as the values of 2 * heads keys.)"""
    return max(1, min(256 // rows, -(-seen // max(128, 8 * heads)), 32))


def talk_attn(q: torch.Tensor, vc: torch.Tensor, inv: torch.Tensor,
              st: StepMeta, tk: Talk) -> torch.Tensor:
    """Talking-heads attention of a step's tokens over their sequences' pages.
    q/out [n, H, P]."""
    n, h, p = q.shape
    g, per, dev = vc.shape[1], st.table.shape[1], q.device
    _dense(q, vc, inv, st.table, tk.knorm, tk.talk, tk.talk16, *tk.rot)
    assert tk.talk.shape == (h, h) and tk.knorm.shape == (p,) and h % g == 0
    out = torch.empty_like(q)
    nrot, r = tk.rot[0].shape[0], 2 * tk.rot[0].shape[1]
    one, tiled = _talk_sizes(tk, g, p)
    cap = (2 * LOG2E * tk.scale / tk.cap, tk.cap * LOG2E,
           max(0.0, tk.cap * LOG2E - 80.0))
    if _f32(q) or not one:
        _call("gt_talk_plain", _f32(q), out, q, vc, inv, st.table, per, st.pos,
              st.slot, tk.knorm, tk.talk, *tk.rot, nrot, n, h, g, p, r,
              tk.chunk, tk.scale, tk.cap)
        return out
    portions = st.talk.get(tk.chunk) if tiled else None
    na = n if portions is None else st.absorbed
    if na:
        nsplit = _talk_splits(na, h, min(st.max_len, tk.chunk))
        ws = torch.empty(na * nsplit * (g * h * p + h), dtype=torch.float32,
                         device=dev) if nsplit > 1 else None
        _call("gt_talk_decode", out, q, vc, inv, st.table, per, st.pos,
              st.slot, ws, tk.knorm, tk.talk, *tk.rot, nrot, na, h, g, p, r,
              tk.chunk, nsplit, *cap)
    if portions is not None:
        kx = torch.empty(2, portions.pages, g, PAGE * p, dtype=q.dtype,
                         device=dev)
        _call("gt_talk_gather", kx[0], kx[1], vc, inv, st.table, per, tk.knorm,
              *tk.rot, nrot, portions.items, portions.items.shape[0], g, p, r)
        lse = torch.empty(n, h, dtype=torch.float32, device=dev)
        _call("gt_talk_lse", lse, q, kx[0], portions.tiles128,
              portions.tiles128.shape[0], h, g, p, tk.chunk, *cap)
        nt = portions.tiles16.shape[0]
        # few tiles: their keys in parts, of 128 or more
        parts = max(1, min(256 // nt, portions.span // 128, 8))
        ws = torch.empty(parts, n - na, h, p, dtype=torch.float32,
                         device=dev) if parts > 1 else None
        _call("gt_talk_prefill", out, q, kx[0], kx[1], lse, tk.talk16,
              portions.tiles16, nt, h, g, p, tk.chunk, *cap, tk.talk16_scale,
              ws, parts, na, n - na)
    return out
