"""Cache and state manager of the serving engine.

A model lists, for every layer run, what it keeps between steps:

* ``PagedKV``      keys and values of an attention, in pages of 64 tokens,
* ``PagedLatent``  latents and shared key columns of a latent attention, one
                 row a token for all heads, in the same pages,
* ``MatrixState``  the state of a recurrent matrix memory, one slot a request,
* ``ConvRing``     the last inputs of a short convolution over time, one slot a
                 request.

All layers share one block table per request (page index -> the same page in
every layer's pool), so the host tracks pages once.  Pages behind every
layer's window that hold no kept first token return to the pool while the
request runs.  One spare page and one spare slot absorb the padding rows of
captured decode graphs.
"""

from dataclasses import dataclass, field
from typing import Dict, List, Optional

import numpy as np
import torch

from ..ops.serving import PAGE_SIZE


class CacheFull(RuntimeError):
    """No page or slot is free for what was asked."""


class Paged:
    """What is kept token by token: a ``window`` (0: every earlier token
    stays visible) and ``keep_first`` tokens that stay visible behind it."""


@dataclass(frozen=True)
class PagedLatent(Paged):
    rank: int            # latent columns
    shared: int          # rotated key columns, shared by all heads
    window: int = 0
    keep_first: int = 0

    def allocate(self, pages, slots, dtype, device):
        return torch.zeros(pages, PAGE_SIZE, self.rank + self.shared,
                           dtype=dtype, device=device)


@dataclass(frozen=True)
class PagedKV(Paged):
    kv_heads: int
    dim: int
    vdim: int
    window: int = 0      # 0: every earlier token stays visible
    keep_first: int = 0  # first tokens that stay visible behind the window

    def allocate(self, pages, slots, dtype, device):
        return (torch.zeros(pages, self.kv_heads, PAGE_SIZE, self.dim,
                            dtype=dtype, device=device),
                torch.zeros(pages, self.kv_heads, PAGE_SIZE, self.vdim,
                            dtype=dtype, device=device))


@dataclass(frozen=True)
class MatrixState:
    heads: int
    dim: int
    vdim: int
    normalized: bool = False  # with a normaliser and a running maximum

    def allocate(self, pages, slots, dtype, device):
        f32 = dict(dtype=torch.float32, device=device)
        S = torch.zeros(slots, self.heads, self.dim, self.vdim, **f32)
        if not self.normalized:
            return S, None, None
        nt = (self.vdim + 31) // 32
        return (S, torch.zeros(slots, self.heads, nt, self.dim, **f32),
                torch.zeros(slots, self.heads, nt, **f32))


@dataclass(frozen=True)
class ConvRing:
    """The input at position p is in place p % taps; a place is read only if
    its request has been there, so a slot needs no clearing."""
    channels: int
    taps: int

    def allocate(self, pages, slots, dtype, device):
        return torch.zeros(slots, self.taps, self.channels, dtype=dtype,
                           device=device)


@dataclass
class RequestState:
    slot: int
    length: int = 0                                # tokens in the cache
    pages: List[int] = field(default_factory=list)  # by position; -1 released
    first_live: int = 0                            # pages before are checked


class CacheManager:
    """Pools on the device, page and slot accounting on the host."""

    def __init__(self, specs, max_tokens: int, max_seqs: int,
                 max_context: Optional[int] = None, dtype=torch.bfloat16,
                 device=None):
        self.specs = specs
        self.num_pages = -(-max_tokens // PAGE_SIZE)
        self.num_slots = max_seqs
        self.max_context = max_context or self.num_pages * PAGE_SIZE
        flat = [s for run in specs for s in run]
        kv = [s for s in flat if isinstance(s, Paged)]
        self.paged = bool(kv)
        # a page may go once it is behind every layer's window
        self.window = max((s.window for s in kv), default=0) \
            if all(s.window > 0 for s in kv) else 0
        self.keep_first = max((s.keep_first for s in kv), default=0)
        self.table_width = -(-self.max_context // PAGE_SIZE) \
            if self.paged else 1
        self.spare_page, self.spare_slot = self.num_pages, self.num_slots
        self._free_pages = list(range(self.num_pages - 1, -1, -1))
        self._free_slots = list(range(self.num_slots - 1, -1, -1))
        self.requests: Dict[object, RequestState] = {}
        self.pools = [[s.allocate(self.num_pages + 1, self.num_slots + 1,
                                  dtype, device) for s in run]
                      for run in specs] if device is not None else None

    # -- accounting ---------------------------------------------------------
    @property
    def free_pages(self) -> int:
        return len(self._free_pages)

    @property
    def free_slots(self) -> int:
        return len(self._free_slots)

    @staticmethod
    def pages_for(tokens: int) -> int:
        return -(-tokens // PAGE_SIZE)

    def admit(self, rid) -> RequestState:
        if rid in self.requests:
            raise ValueError(f"request {rid!r} is already live")
        if not self._free_slots:
            raise CacheFull("no free slot")
        st = RequestState(slot=self._free_slots.pop())
        self.requests[rid] = st
        return st

    def _release_behind(self, st: RequestState):
        """Return pages that no later token can see."""
        if not self.window:
            return
        first_visible = st.length - self.window + 1
        while (st.first_live + 1) * PAGE_SIZE <= first_visible:
            i = st.first_live
            if i * PAGE_SIZE >= self.keep_first and st.pages[i] >= 0:
                self._free_pages.append(st.pages[i])
                st.pages[i] = -1
            st.first_live += 1

    def extend(self, rid, tokens: int) -> RequestState:
        """Make room for the request's next tokens (all or nothing)."""
        st = self.requests[rid]
        if st.length + tokens > self.max_context:
            raise CacheFull(f"{st.length + tokens} tokens exceed the context "
                            f"limit {self.max_context}")
        if self.paged:
            self._release_behind(st)
            need = self.pages_for(st.length + tokens) - len(st.pages)
            if need > len(self._free_pages):
                raise CacheFull(f"{need} pages needed, "
                                f"{len(self._free_pages)} free")
            for _ in range(need):
                st.pages.append(self._free_pages.pop())
        return st

    def free(self, rid):
        st = self.requests.pop(rid)
        self._free_pages.extend(p for p in reversed(st.pages) if p >= 0)
        self._free_slots.append(st.slot)

    def table_row(self, st: RequestState, out: np.ndarray):
        """The block-table row; places without a page name the spare one."""
        out[:] = self.spare_page
        if st.pages:
            row = np.asarray(st.pages, dtype=np.int32)
            out[:len(row)] = np.where(row < 0, self.spare_page, row)
