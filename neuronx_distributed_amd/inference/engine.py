"""Serving engine: one step runs a ragged batch through a model.

A step brings the next tokens of any number of live requests — portions of
prompts beside single decoded tokens — and runs them together from the
cache pages and state slots that earlier steps left.  Portions come first in
the packed batch, single tokens after them, so each kind goes through its
own kernels.  Steps made of single tokens only replay a hipGraph captured
per batch-size bucket.

A model is served when it has ``cache_specs()`` and
``forward_ragged(batch, pools)``; ``max_positions``, if it has one, bounds
the context.
"""

from dataclasses import dataclass
from typing import Dict, List, Optional, Sequence

import numpy as np
import torch

from ..ops import serving as sv
from .paged_cache import (PAGE_SIZE, CacheManager, PagedLatent,
                          RequestState)

TILE_ROWS = 128


@dataclass
class StepEntry:
    """Next tokens of one request; ``want`` are the places among them whose
    logits are asked for."""
    id: object
    tokens: Sequence[int]
    want: Sequence[int] = ()


@dataclass
class RaggedBatch:
    """Device view of a packed step (all int32)."""
    tokens: torch.Tensor       # (T,)
    pos: torch.Tensor          # (T,)
    seq: torch.Tensor          # (T,) row of the block table
    block_table: torch.Tensor  # (R, width)
    tiles: torch.Tensor        # (n, 4) query tiles of the portions
    portions: torch.Tensor     # (n, 4) slot, first row, rows, context
    chunks: torch.Tensor       # (n, 4) chunks of the portions
    chunk_first: torch.Tensor  # (portions + 1,) first chunk of each
    singles: torch.Tensor      # (n, 4) like portions, for single tokens
    want: torch.Tensor         # (W,) rows whose logits are computed
    portion_tokens: int        # rows [0, portion_tokens) belong to portions
    max_keys: int              # no row sees more keys than this
    # window -> keys of the portions, for latent attention; none when the
    # portions are so short that they run like single tokens
    spans: Dict[int, sv.KeySpans]


class _Layout:
    """Places of the batch's arrays in one int32 buffer (one upload)."""

    def __init__(self, T, portion_tokens, R, n_tiles, n_portions, n_chunks,
                 n_singles, n_want, width, span_pages={}):
        self.portion_tokens = portion_tokens
        self.windows = list(span_pages)
        self.at, n = {}, 0
        spans = [a for w, pages in span_pages.items()
                 for a in (((w, "pages"), (pages,)),
                           ((w, "table"), (n_portions, width)))]
        for name, shape in (*spans, ("tokens", (T,)), ("pos", (T,)), ("seq", (T,)),
                            ("tiles", (n_tiles, 4)),
                            ("portions", (n_portions, 4)),
                            ("chunks", (n_chunks, 4)),
                            ("chunk_first", (n_portions + 1,)),
                            ("singles", (n_singles, 4)),
                            ("want", (n_want,)),
                            ("block_table", (R, width))):
            size = int(np.prod(shape))
            self.at[name] = (n, size, shape)
            n += -(-size // 4) * 4
        self.size = max(n, 4)

    def views(self, buf):
        return {k: buf[o:o + s].reshape(shape)
                for k, (o, s, shape) in self.at.items()}

    def batch(self, buf, max_keys) -> RaggedBatch:
        v = self.views(buf)
        spans = {w: sv.KeySpans(v.pop((w, "pages")), v.pop((w, "table")))
                 for w in self.windows}
        return RaggedBatch(portion_tokens=self.portion_tokens,
                           max_keys=max_keys, spans=spans, **v)


class InferenceEngine:
    def __init__(self, model, max_tokens: int, max_seqs: int,
                 max_context: Optional[int] = None, use_graphs: bool = True):
        for name in ("cache_specs", "forward_ragged"):
            if not hasattr(model, name):
                raise TypeError(f"{type(model).__name__} has no {name}()")
        p = next(model.parameters())
        if not p.is_cuda:
            raise RuntimeError("the serving engine runs on the GPU only")
        limit = getattr(model, "max_positions", None)
        if limit is not None:
            if max_context is not None and max_context > limit:
                raise ValueError(f"a context of {max_context} tokens; the "
                                 f"model has {limit} positions")
            max_context = min(limit, max_context or
                              CacheManager.pages_for(max_tokens) * PAGE_SIZE)
        self.model = model
        self.device = p.device
        specs = model.cache_specs()
        self.cache = CacheManager(specs, max_tokens, max_seqs, max_context,
                                  dtype=p.dtype, device=self.device)
        self._latent_windows = sorted({
            s.window for run in specs for s in run
            if isinstance(s, PagedLatent)})
        self.max_seqs = max_seqs
        self.use_graphs = use_graphs
        self._graphs: Dict[int, tuple] = {}
        self._pool = None

    # -- requests -----------------------------------------------------------
    def finish(self, rid):
        """Give back the pages and the slot of a request."""
        self.cache.free(rid)

    @torch.no_grad()
    def step(self, entries: Sequence[StepEntry]) -> Optional[torch.Tensor]:
        """Run the entries as one batch.  Returns float32 logits
        (wanted, vocab) in the order of the entries and of their ``want``,
        or None if nothing is wanted.  A new id is admitted."""
        entries = [e for e in entries if len(e.tokens)]
        if not entries:
            return None
        if len({e.id for e in entries}) != len(entries):
            raise ValueError("a request has two entries in one step")
        for e in entries:
            if any(not 0 <= w < len(e.tokens) for w in e.want):
                raise ValueError(f"request {e.id!r} wants a place outside "
                                 "its tokens")
            lo, hi = min(e.tokens), max(e.tokens)
            if lo < 0 or hi >= self.model.config.vocab_size:
                raise ValueError(f"request {e.id!r} has a token outside the "
                                 "vocabulary")
        admitted = []
        try:
            for e in entries:
                if e.id not in self.cache.requests:
                    self.cache.admit(e.id)
                    admitted.append(e.id)
            states = [self.cache.extend(e.id, len(e.tokens))
                      for e in entries]
        except Exception:
            for rid in admitted:
                self.cache.free(rid)
            raise
        if self.use_graphs and all(len(e.tokens) == 1 for e in entries):
            logits = self._replay(entries, states)
        else:
            logits = self._eager(entries, states)
        for e, st in zip(entries, states):
            st.length += len(e.tokens)
        return logits

    # -- batches ------------------------------------------------------------
    def _eager(self, entries: List[StepEntry], states: List[RequestState]):
        order = sorted(range(len(entries)),
                       key=lambda i: len(entries[i].tokens) == 1)
        n_port = sum(len(e.tokens) > 1 for e in entries)
        row_of = {}
        T = 0
        for i in order:
            row_of[i] = T
            T += len(entries[i].tokens)
        portion_tokens = sum(len(e.tokens) for e in entries
                             if len(e.tokens) > 1)
        n_tiles = sum(-(-len(e.tokens) // TILE_ROWS) for e in entries
                      if len(e.tokens) > 1)
        want = [row_of[i] + w for i, e in enumerate(entries) for w in e.want]
        portions = [(states[i].slot, row_of[i], len(entries[i].tokens),
                     states[i].length) for i in order[:n_port]]
        chunks, first = sv.chunk_table(portions)
        spans = self._spans(portions, [states[i] for i in order[:n_port]])
        lay = _Layout(T, portion_tokens, len(entries), n_tiles, n_port,
                      len(chunks), len(entries) - n_port, len(want),
                      self.cache.table_width,
                      {w: len(pages) for w, (pages, _) in spans.items()})
        host = np.zeros(lay.size, dtype=np.int32)
        v = lay.views(host)
        for w, (pages, table) in spans.items():
            v[w, "pages"][:] = pages
            v[w, "table"][:] = table
        v["want"][:] = want
        v["chunks"][:] = np.asarray(chunks, dtype=np.int32).reshape(-1, 4)
        v["chunk_first"][:] = first
        tile = 0
        for s, i in enumerate(order):
            e, st, r0 = entries[i], states[i], row_of[i]
            n = len(e.tokens)
            v["tokens"][r0:r0 + n] = e.tokens
            v["pos"][r0:r0 + n] = np.arange(st.length, st.length + n)
            v["seq"][r0:r0 + n] = s
            self.cache.table_row(st, v["block_table"][s])
            seg = (st.slot, r0, n, st.length)
            if s < n_port:
                v["portions"][s] = seg
                for q in range(0, n, TILE_ROWS):
                    v["tiles"][tile] = (s, r0 + q, min(TILE_ROWS, n - q),
                                        st.length + q)
                    tile += 1
            else:
                v["singles"][s - n_port] = seg
        max_keys = max(st.length + len(e.tokens)
                       for e, st in zip(entries, states))
        buf = torch.from_numpy(host).to(self.device)
        return self.model.forward_ragged(lay.batch(buf, max_keys),
                                         self.cache.pools)

    def _spans(self, portions, states):
        """Host form of the portions' key spans for every latent window."""
        if max((n for _, _, n, _ in portions), default=0) < \
                sv.EXPAND_MIN_TOKENS or not self._latent_windows:
            return {}
        rows = np.zeros((len(states), self.cache.table_width), dtype=np.int32)
        for st, row in zip(states, rows):
            self.cache.table_row(st, row)
        return {w: sv.key_spans(portions, rows, w)
                for w in self._latent_windows}

    def _bucket(self, n: int) -> int:
        b = 1
        while b < n:
            b *= 2
        return min(b, self.max_seqs)

    def _fill_singles(self, v, entries, states, bucket):
        """Rows past the entries are padding: position 0 of the spare slot
        and the spare page."""
        v["tokens"][:] = 0
        v["pos"][:] = 0
        v["seq"][:] = np.arange(bucket)
        v["want"][:] = np.arange(bucket)
        v["block_table"][:] = self.cache.spare_page
        v["singles"][:, 0] = self.cache.spare_slot
        v["singles"][:, 1] = np.arange(bucket)
        v["singles"][:, 2] = 1
        v["singles"][:, 3] = 0
        for s, (e, st) in enumerate(zip(entries, states)):
            v["tokens"][s] = e.tokens[0]
            v["pos"][s] = st.length
            v["singles"][s, 0] = st.slot
            v["singles"][s, 3] = st.length
            self.cache.table_row(st, v["block_table"][s])

    def _capture(self, bucket: int):
        """Capture one decode step of ``bucket`` rows; the warm-up runs on
        padding rows only."""
        lay = _Layout(bucket, 0, bucket, 0, 0, 0, bucket, bucket,
                      self.cache.table_width)
        host = np.zeros(lay.size, dtype=np.int32)
        self._fill_singles(lay.views(host), [], [], bucket)
        buf = torch.from_numpy(host).to(self.device)
        batch = lay.batch(buf, self.cache.max_context)
        side = torch.cuda.Stream()
        side.wait_stream(torch.cuda.current_stream())
        with torch.cuda.stream(side):
            for _ in range(2):
                self.model.forward_ragged(batch, self.cache.pools)
        torch.cuda.current_stream().wait_stream(side)
        torch.cuda.synchronize()
        g = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g, pool=self._pool):
            logits = self.model.forward_ragged(batch, self.cache.pools)
        if self._pool is None:
            self._pool = g.pool()
        self._graphs[bucket] = (g, lay, host, buf, logits)
        return self._graphs[bucket]

    def _replay(self, entries, states):
        bucket = self._bucket(len(entries))
        g, lay, host, buf, logits = (self._graphs.get(bucket)
                                     or self._capture(bucket))
        self._fill_singles(lay.views(host), entries, states, bucket)
        buf.copy_(torch.from_numpy(host))
        g.replay()
        rows = [s for s, e in enumerate(entries) for _ in e.want]
        if not rows:
            return None
        if rows == list(range(len(rows))):
            return logits[:len(rows)].clone()
        return logits[torch.tensor(rows, device=self.device)]
