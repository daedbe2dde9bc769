"""ctypes binding to libgridllm_hybrid.so: the gfx950 kernels of the
layer-list models (csrc/gridllm_hybrid.hip). Same contract as hip_ops:
launches go onto torch's current stream, a missing library raises, shapes are
checked on the host before a launch.

Every function here has a CPU counterpart of the same signature in
reference_hybrid; ops.hybrid picks one by device.
"""

from __future__ import annotations

import ctypes
import os
from typing import Optional

import torch
import torch.nn.functional as F

from gridllm_amd.ops.build import lib_path
from gridllm_amd.ops.hip_ops import (HipExtensionMissing, _check,
                                     _check_range, _ptr, _stream)
from gridllm_amd.ops.reference import Glu
from gridllm_amd.ops.reference_hybrid import StepMeta

_lib: Optional[ctypes.CDLL] = None
PAGE = 64

# argument kinds of each entry point after the stream: p pointer, i int,
# l long, f float
_SIGS = {
    "gh_embed_pos": "ippppppiiii",
    "gh_post_norm": "ippppipfiiif",
    "gh_norm_rows": "ippppfiiif",
    "gh_glu_f32": "pplifff",
    "gh_proj_f32": "ppppiii",
    "gh_qknorm_kv": "ipppppippiiiiiiffi",
    "gh_paged_decode": "pppppipppiiiiifppi",
    "gh_paged_prefill": "pppppipiiiifppi",
    "gh_attn_rows_f32": "pppppippiiiifppi",
    "gh_mlstm_step": "ippppppppiiiiiffi",
    "gh_mlstm_out": "ipppppppppiiiiiiiiff",
    "gh_mlstm_chunks": "pppppppppiiiiiiff",
    "gh_moe_route": "pppppppiiiii",
    "gh_moe_gemm": "iipppppiiiii",
}
_KINDS = {"p": ctypes.c_void_p, "i": ctypes.c_int, "l": ctypes.c_long,
          "f": ctypes.c_float}


def _load() -> ctypes.CDLL:
    global _lib
    if _lib is None:
        path = lib_path("hybrid")
        if not os.path.exists(path):
            raise HipExtensionMissing(
                f"GridLLM HIP kernel library not found at {path}. Build it "
                "with: python -m gridllm_amd.ops.build (this is required on "
                "GPU machines; there is no eager fallback).")
        lib = ctypes.CDLL(path)
        for name, sig in _SIGS.items():
            fn = getattr(lib, name)
            fn.argtypes = [ctypes.c_void_p] + [_KINDS[c] for c in sig]
            fn.restype = ctypes.c_int
        _lib = lib
    return _lib


def _call(name: str, *args) -> None:
    args = [_ptr(a) if a is None or isinstance(a, torch.Tensor) else a
            for a in args]
    _check(getattr(_load(), name)(_stream(), *args), name)


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


def embed_pos(tok: torch.Tensor, pos: torch.Tensor, emb: torch.Tensor,
              ptab: torch.Tensor) -> tuple[torch.Tensor, torch.Tensor]:
    """f32 residual embed[tok] + ptab[pos], and its copy in the weights' type
    (the same tensor if that is f32)."""
    n, w = tok.shape[0], emb.shape[1]
    _dense(tok, pos, emb, ptab)
    x = torch.empty(n, w, dtype=torch.float32, device=tok.device)
    f = _f32(emb)
    xb = x if f else torch.empty(n, w, dtype=emb.dtype, device=tok.device)
    _call("gh_embed_pos", f, x, None if f else xb, emb, ptab, tok, pos, n, w,
          emb.shape[0], ptab.shape[0])
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


def qknorm_kv(qkv: torch.Tensor, kc: torch.Tensor, vc: torch.Tensor,
              st: StepMeta, heads: int, kv_heads: int, dim: int, eps: float,
              coef: float, every: int) -> torch.Tensor:
    """Unit-RMS q (with temperature) -> [n, heads, P]; unit-RMS k and v go to
    the pages of kc / vc [pages, kv_heads, 64, P]."""
    n, p = qkv.shape[0], kc.shape[3]
    _dense(qkv, kc, vc, st.table)
    assert qkv.shape[1] >= (heads + 2 * kv_heads) * p
    _check_range("qknorm_kv.slot", st.slot, st.table.shape[0])
    q = torch.empty(n, heads, p, dtype=qkv.dtype, device=qkv.device)
    _call("gh_qknorm_kv", _f32(qkv), qkv, q, kc, vc, st.table,
          st.table.shape[1], st.pos, st.slot, n, heads, kv_heads, p,
          qkv.shape[1], dim, eps, coef, every)
    return q


def paged_attn(q: torch.Tensor, kc: torch.Tensor, vc: torch.Tensor,
               st: StepMeta, scale: float, sink: Optional[torch.Tensor],
               gate: Optional[torch.Tensor]) -> torch.Tensor:
    """Causal attention of a step's tokens over their sequences' pages.
    q/out [n, heads, P]; sink [heads] f32; gate [n, >= heads] (a column view
    of the projection rows is fine)."""
    n, h, p = q.shape
    g = kc.shape[1]
    _dense(q, kc, vc, st.table, sink)
    out = torch.empty_like(q)
    ld = 0
    if gate is not None:
        assert gate.stride(1) == 1 and gate.dtype == q.dtype
        ld = gate.stride(0)
    per = st.table.shape[1]
    if _f32(q):
        _call("gh_attn_rows_f32", out, q, kc, vc, st.table, per, st.pos,
              st.slot, n, h, g, p, scale, sink, gate, ld)
        return out
    if st.nd:
        groups = h // max(d for d in range(1, 9) if (h // g) % d == 0)
        nsplit = max(1, min(512 // max(1, st.nd * groups),
                            (st.max_len + 255) // 256, 32))
        ws = torch.empty(st.nd * h * nsplit * (p + 2), dtype=torch.float32,
                         device=q.device) if nsplit > 1 else None
        _call("gh_paged_decode", out, q, kc, vc, st.table, per, st.pos,
              st.slot, ws, st.nd, h, g, p, nsplit, scale, sink, gate, ld)
    if st.tiles is not None:
        _call("gh_paged_prefill", out, q, kc, vc, st.table, per, st.tiles,
              st.tiles.shape[0], h, g, p, scale, sink, gate, ld)
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
        _call("gh_mlstm_step", f, o, S, m, qkv, gates, segs, st.pos, st.slot,
              nseg, h, dk, dv, ld, qscale, cap, rpb)
    nplain = 0
    if not f and st.chunks is not None:
        nplain = n - st.nd
        nch = st.chunks.shape[0]
        ds = torch.empty(nch, h, dv + 1, dk, dtype=torch.float32,
                         device=qkv.device)
        scal = torch.empty(nch, h, 4, dtype=torch.float32, device=qkv.device)
        _call("gh_mlstm_chunks", o, S, m, ds, scal, qkv, gates, st.chunks,
              st.chunk_segs, nch, st.chunk_segs.shape[0], h, dk, dv, ld,
              qscale, cap)
    out = torch.empty(n, h * dv, dtype=qkv.dtype, device=qkv.device)
    _call("gh_mlstm_out", f, out, o, m, qkv, gates, segs, st.pos, st.slot,
          norm, nseg, st.nd, nplain, h, dk, dv, ld, vdim, cap, eps)
    return out


# up to this many (token, expert) pairs, mostly of different experts, the
# 16-row kernel fills the chip better than 128 x 128 tiles do
_FEW_PAIRS = 64


def moe(x: torch.Tensor, logits: torch.Tensor, up: torch.Tensor,
        down: torch.Tensor, top: int) -> tuple[torch.Tensor, torch.Tensor]:
    """Routed experts with squared ReLU. x [n, W]; logits f32 [n, E];
    up [E, F, W]; down [E, W, F]. Returns the chosen experts' outputs
    [n * top, W] in pair order and their weights f32 [n, top]."""
    n, w = x.shape
    e, ff = up.shape[0], up.shape[1]
    _dense(x, logits, up, down)
    dev, f = x.device, _f32(x)
    pairs = n * top
    bm = 16 if f or pairs <= _FEW_PAIRS else 128
    max_tiles = min(pairs, e + pairs // bm)
    ints = torch.empty(3 * pairs, dtype=torch.int32, device=dev)
    idx, rank, order = ints[:pairs], ints[pairs:2 * pairs], ints[2 * pairs:]
    counts = torch.zeros(e, dtype=torch.int32, device=dev)
    tiles = torch.empty(max_tiles + 1, 4, dtype=torch.int32, device=dev)
    wt = torch.empty(n, top, dtype=torch.float32, device=dev)
    _call("gh_moe_route", idx, wt, rank, counts, order, tiles, logits, n, e,
          top, bm, max_tiles)
    act = torch.empty(pairs, ff, dtype=x.dtype, device=dev)
    _call("gh_moe_gemm", f, 1, act, x, up, tiles, order, top, ff, w, bm,
          max_tiles)
    ye = torch.empty(pairs, w, dtype=x.dtype, device=dev)
    _call("gh_moe_gemm", f, 0, ye, act, down, tiles, order, top, w, ff, bm,
          max_tiles)
    return ye, wt
