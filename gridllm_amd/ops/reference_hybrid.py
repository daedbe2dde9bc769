"""Pure-PyTorch execution of the layer-list ops on the CPU (no GPU in CI),
function for function the signatures of hip_hybrid, and the description of a
step that both take."""

from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch
import torch.nn.functional as F

PAGE = 64


@dataclass
class StepMeta:
    """The tokens of one step: `nd` decode rows (one token of a sequence
    each), then prompt portions. Everything but nd and max_len lives on the
    device.

    tiles      [*, 8] {first token, length, slot, first row, start} per 128
               rows of a portion (attention)
    chunks     [*, 4] {first token, length, portion} per 64 tokens, and
    chunk_segs [*, 4] {slot, start, first chunk, chunks} per portion (mLSTM)
    segs       [*, 4] {first token, length, slot, start} of every entry, decode
               rows included; what the token-by-token paths walk. None: all
               entries are decode rows.
    """
    nd: int
    pos: torch.Tensor            # [n] int32
    slot: torch.Tensor           # [n] int32
    table: torch.Tensor          # [slots, pages per slot] int32
    max_len: int                 # bound of any sequence's length
    tiles: Optional[torch.Tensor] = None
    chunks: Optional[torch.Tensor] = None
    chunk_segs: Optional[torch.Tensor] = None
    segs: Optional[torch.Tensor] = None

    def entries(self) -> list:
        """(first token, length, slot, start) of every entry, on the host."""
        if self.segs is not None:
            return [tuple(r) for r in self.segs.tolist()]
        return [(i, 1, s, p) for i, (s, p) in enumerate(
            zip(self.slot.tolist(), self.pos.tolist()))]


def embed_pos(tok, pos, emb, ptab):
    x = emb[tok].float() + ptab[pos.long()].float()
    return x, (x if emb.dtype == torch.float32 else x.to(emb.dtype))


def _norm(y, w, w_off, width, eps):
    rs = torch.rsqrt(y.pow(2).sum(-1, keepdim=True) / width + eps)
    return y * rs * (w_off + w)


def post_norm(x, xb, y, w, w_off, width, eps, pair_w=None):
    y = y.float()
    if pair_w is not None:
        y = (y.view(*pair_w.shape, -1) * pair_w.unsqueeze(-1)).sum(1)
    x += _norm(y, w, w_off, width, eps)
    if xb is not x:
        xb.copy_(x)


def norm_rows(x, rows, w, w_off, width, eps, dtype):
    z = x if rows is None else x[rows.long()]
    return _norm(z, w, w_off, width, eps).to(dtype)


def proj_f32(x, w, bias=None):
    return F.linear(x.float(), w.float(), bias)


def _rows_of(cache, table, slot, lo, hi):
    """Rows lo..hi-1 of a slot as (page, offset) index pairs."""
    p = torch.arange(lo, hi)
    return table[slot, p // PAGE].long(), p % PAGE


def qknorm_kv(qkv, kc, vc, st, heads, kv_heads, dim, eps, coef, every):
    n, p = qkv.shape[0], kc.shape[3]
    cols = qkv[:, :(heads + 2 * kv_heads) * p].float().view(n, -1, p)
    q, k, v = cols.split([heads, kv_heads, kv_heads], dim=1)

    def unit(z):
        return z * torch.rsqrt(z.pow(2).sum(-1, keepdim=True) / dim + eps)

    steps = torch.div(st.pos + 1, every, rounding_mode="floor").float()
    q = unit(q) * (1 + coef * torch.log(steps + 1)).view(n, 1, 1)
    k = unit(k)
    page = st.table[st.slot.long(), (st.pos // PAGE).long()].long()
    off = (st.pos % PAGE).long()
    kc[page, :, off] = k.to(kc.dtype)
    vc[page, :, off] = v.to(vc.dtype)
    return q.to(qkv.dtype)


def paged_attn(q, kc, vc, st, scale, sink, gate):
    n, h, p = q.shape
    g = kc.shape[1]
    out = torch.empty_like(q)
    for off, ln, slot, start in st.entries():
        total = start + ln
        page, row = _rows_of(kc, st.table, slot, 0, total)
        k = kc[page, :, row].float().repeat_interleave(h // g, dim=1)
        v = vc[page, :, row].float().repeat_interleave(h // g, dim=1)
        s = torch.einsum("thd,shd->hts", q[off:off + ln].float(), k) * scale
        ahead = torch.arange(total).view(1, 1, -1) > \
            torch.arange(start, total).view(1, -1, 1)
        s = s.masked_fill(ahead, float("-inf"))
        if sink is not None:
            s = torch.cat([s, sink.view(h, 1, 1).expand(h, ln, 1)], dim=-1)
        w = torch.softmax(s, dim=-1)[..., :total]
        out[off:off + ln] = torch.einsum("hts,shd->thd", w, v).to(q.dtype)
    if gate is not None:
        out *= torch.sigmoid(gate[:, :h].float()).unsqueeze(-1).to(q.dtype)
    return out


def mlstm(qkv, gates, S, m, norm, st, dim, vdim, cap, eps):
    n = qkv.shape[0]
    h, dv, dk = S.shape[1], S.shape[2] - 1, S.shape[3]
    q, k, v, g = qkv[:, :h * 2 * (dk + dv)].float().split(
        [h * dk, h * dk, h * dv, h * dv], dim=1)
    q = q.view(n, h, dk) * dim ** -0.5
    k = k.view(n, h, dk)
    v = F.pad(v.view(n, h, dv), (0, 1), value=1.0)   # last row: normaliser
    gi = cap * torch.tanh(gates[:, :h] / cap)
    gf = F.logsigmoid(cap * torch.tanh(gates[:, h:] / cap))
    o = torch.empty(n, h, dv)
    for off, ln, slot, start in st.entries():
        s, mm = S[slot], m[slot]
        if start == 0:
            s, mm = torch.zeros_like(s), torch.zeros_like(mm)
        for t in range(off, off + ln):
            m2 = torch.maximum(gf[t] + mm, gi[t])
            keep, put = torch.exp(gf[t] + mm - m2), torch.exp(gi[t] - m2)
            mm = m2
            s = keep.view(h, 1, 1) * s + put.view(h, 1, 1) * \
                v[t].unsqueeze(2) * k[t].unsqueeze(1)
            r = torch.matmul(s, q[t].unsqueeze(2)).squeeze(2)
            den = torch.maximum(r[:, dv].abs(), torch.exp(-mm)) + 1e-6
            o[t] = r[:, :dv] / den.view(h, 1)
        S[slot], m[slot] = s, mm
    o = o * torch.rsqrt(o.pow(2).sum(-1, keepdim=True) / vdim + eps)
    return (o.reshape(n, -1) * norm * torch.sigmoid(g)).to(qkv.dtype)


def moe(x, logits, up, down, top):
    val, idx = torch.topk(logits, top, dim=-1)
    wt = torch.softmax(val, dim=-1)
    flat = idx.reshape(-1)
    xs = x.repeat_interleave(top, dim=0).float()
    ye = torch.empty(flat.shape[0], x.shape[1], dtype=x.dtype)
    for e in torch.unique(flat).tolist():
        r = (flat == e).nonzero().squeeze(1)
        a = torch.relu(xs[r] @ up[e].float().T) ** 2
        ye[r] = (a @ down[e].float().T).to(x.dtype)
    return ye, wt
