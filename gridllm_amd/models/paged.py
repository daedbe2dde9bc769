"""Cache and state manager of layer-list models.

Two kinds of memory per sequence. Attention layers share one pool of pages of
64 tokens (one page id holds a sequence's 64 tokens in every attention layer):
keys and values, one row of latent and rotated key part per token, or (where
keys are made from the values) values and the inverse of their rms. Recurrent
layers have a state of fixed size per slot. A sequence is a slot: a row of the
page table plus its states.

Pages are taken when a sequence grows into them. `alloc(tokens)` sets aside as
many as the sequence may come to need, so that growing never fails for a
sequence admitted with its bound; `alloc(0)` promises nothing and grows as long
as there are pages. The interface is the slot cache's (alloc, free, n_free,
reserve, seq_lens), so engine and batcher treat both alike; n_free counts how
many more sequences of full length fit.

All bookkeeping is on the host; the table's changes go up in one scatter per
step, and only in steps in which a sequence enters a new page.
"""

from __future__ import annotations

from typing import Callable, Optional, Sequence, Union

import numpy as np
import torch

from gridllm_amd.models.registry import (AttentionMixer, GlaMixer,
                                         HybridSpec, LatentMixer,
                                         LightningMixer, MlstmMixer,
                                         ParallelMixer, TalkingMixer)

PAGE = 64


def pad64(n: int) -> int:
    return (n + 63) // 64 * 64


def _next_of(sizes: tuple, n: int, what: str) -> int:
    for p in sizes:
        if n <= p:
            return p
    raise ValueError(f"{what} of {n}: more than {sizes[-1]} is not supported")


def head_pad(mixer: Union[AttentionMixer, LatentMixer, TalkingMixer]) -> int:
    """Head size that the attention kernels run at: keys and values padded to
    the next of 64, 128, 256."""
    return _next_of((64, 128, 256),
                    max(mixer.dim, getattr(mixer, "vdim", 0)),
                    "attention heads")


def latent_pad(mixer: LatentMixer) -> tuple[int, int]:
    """Latent and rotated size that the latent-attention kernels run at; a
    cached row is their sum."""
    return (_next_of((64, 128, 256, 512), mixer.kv_rank, "latents"),
            _next_of((64, 128), mixer.rot_dim, "rotated key parts"))


def rotated_pad(mixer: TalkingMixer) -> int:
    """Leading coordinates of a head that the talking-heads kernels treat as
    rotated."""
    p = head_pad(mixer)
    return next(r for r in ((64, 256) if p == 256 else (32, 64, p))
                if mixer.rot_dims <= r)


class PagedCache:
    def __init__(self, spec: HybridSpec, slots: int, max_seq: int,
                 device: torch.device, dtype: torch.dtype,
                 pool_tokens: int = 0,
                 upload: Optional[Callable] = None):
        self.slots = slots
        self.max_seq = max_seq
        self.device = device
        self.per_slot = -(-max_seq // PAGE)
        pages = -(-pool_tokens // PAGE) if pool_tokens else \
            slots * self.per_slot
        self.pages = pages
        # page 0 belongs to nobody: unset table entries point to it, and the
        # padding rows of a captured decode step write there
        self.k: list[Optional[torch.Tensor]] = []
        self.v: list[Optional[torch.Tensor]] = []
        self.lat: list[Optional[torch.Tensor]] = []
        self.inv: list[Optional[torch.Tensor]] = []
        self.S: list[Optional[torch.Tensor]] = []
        self.m: list[Optional[torch.Tensor]] = []
        for ly in spec.layers:
            mx = rec = ly.mixer
            if isinstance(mx, ParallelMixer):     # pages and a state
                mx, rec = mx.left, mx.right
            k = v = lat = inv = s = m = None
            if isinstance(mx, AttentionMixer):
                shape = (pages + 1, mx.kv_heads, PAGE, head_pad(mx))
                k = torch.zeros(shape, dtype=dtype, device=device)
                v = torch.zeros(shape, dtype=dtype, device=device)
            elif isinstance(mx, LatentMixer):
                lat = torch.zeros(pages + 1, PAGE, sum(latent_pad(mx)),
                                  dtype=dtype, device=device)
            elif isinstance(mx, TalkingMixer):
                shape = (pages + 1, mx.kv_heads, PAGE)
                v = torch.zeros(*shape, head_pad(mx), dtype=dtype,
                                device=device)
                inv = torch.zeros(shape, device=device)
            if isinstance(rec, (GlaMixer, LightningMixer)):
                s = torch.zeros(slots, rec.heads, pad64(rec.vdim),
                                pad64(rec.dim), device=device)
            elif isinstance(rec, MlstmMixer):
                s = torch.zeros(slots, rec.heads, pad64(rec.vdim) + 1,
                                pad64(rec.dim), device=device)
                m = torch.zeros(slots, rec.heads, device=device)
            self.k.append(k)
            self.v.append(v)
            self.lat.append(lat)
            self.inv.append(inv)
            self.S.append(s)
            self.m.append(m)
        self.table = torch.zeros(slots, self.per_slot, dtype=torch.int32,
                                 device=device)
        self.seq_lens = torch.zeros(slots, dtype=torch.int32, device=device)
        self.lens = np.zeros(slots, dtype=np.int64)     # host's view
        self._upload = upload
        self._free = list(range(slots))
        self._free_pages = list(range(pages, 0, -1))
        self._held: list[list[int]] = [[] for _ in range(slots)]
        self._bound = [0] * slots          # pages set aside at admission
        self._owed = 0                     # of these, not taken yet
        self._changes: list[tuple[int, int]] = []

    # -- sequences ---------------------------------------------------------

    def reserve(self, slot: int) -> None:
        """Remove a slot from the allocatable ones (hipGraph scratch slot: all
        its table entries stay on page 0)."""
        if slot in self._free:
            self._free.remove(slot)

    def alloc(self, tokens: Optional[int] = None) -> int:
        """A slot, with pages set aside for `tokens` (None: full length)."""
        need = self.per_slot if tokens is None else \
            -(-min(tokens, self.max_seq) // PAGE)
        if not self._free:
            raise RuntimeError("KV cache: no free slots")
        if need > len(self._free_pages) - self._owed:
            raise RuntimeError(
                f"KV cache: {need} pages wanted, "
                f"{len(self._free_pages) - self._owed} not spoken for")
        slot = self._free.pop()
        self._bound[slot] = need
        self._owed += need
        self.lens[slot] = 0
        return slot

    def free(self, slot: int) -> None:
        held = self._held[slot]
        self._owed -= max(0, self._bound[slot] - len(held))
        self._bound[slot] = 0
        self._free_pages.extend(reversed(held))
        held.clear()
        self.lens[slot] = 0
        self._free.append(slot)

    def _grow(self, slot: int, length: int) -> None:
        if length > self.max_seq:
            raise RuntimeError(f"sequence of {length} tokens in a cache for "
                               f"{self.max_seq}")
        held = self._held[slot]
        while len(held) * PAGE < length:
            inside = len(held) < self._bound[slot]
            if not inside and len(self._free_pages) <= self._owed:
                raise RuntimeError("KV cache: out of pages")
            page = self._free_pages.pop()
            self._owed -= inside
            self._changes.append((slot * self.per_slot + len(held), page))
            held.append(page)
        self.lens[slot] = length

    def extend(self, slots: Sequence[int], counts: Sequence[int]) -> None:
        """The sequences of `slots` take `counts` more tokens: assign pages
        and bring the device's table up to date."""
        for s, c in zip(slots, counts):
            self._grow(s, int(self.lens[s]) + c)
        self._flush()

    def prepare_decode(self, slots: Sequence[int]) -> None:
        """One more token for each of `slots`; to be called ahead of a decode
        step (the step itself runs on the device's lengths alone)."""
        idx = np.asarray(slots, dtype=np.int64)
        ln = self.lens[idx]
        edge = (ln % PAGE == 0) | (ln >= self.max_seq)
        for s in idx[edge]:
            self._grow(int(s), int(self.lens[s]) + 1)
        self.lens[idx[~edge]] += 1
        self._flush()

    def _flush(self) -> None:
        if not self._changes:
            return
        ch = np.asarray(self._changes, dtype=np.int64).T
        self._changes = []
        dev = self._upload(ch) if self._upload else \
            torch.from_numpy(np.ascontiguousarray(ch)).to(self.device)
        self.table.view(-1).index_copy_(0, dev[0], dev[1].to(torch.int32))

    @property
    def n_free(self) -> int:
        spare = len(self._free_pages) - self._owed
        return min(len(self._free), spare // self.per_slot)

    def bytes(self) -> int:
        return sum(t.numel() * t.element_size()
                   for ts in (self.k, self.v, self.lat, self.inv, self.S,
                              self.m)
                   for t in ts if t is not None)
