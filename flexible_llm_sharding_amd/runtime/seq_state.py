"""Per-request state of a hybrid stack: K/V pages for its attention layers, slots for the state
of its recurrent layers.

The scoring engine's :class:`~.prefix_cache.PrefixKVCache` keeps whole prefixes and suffixes of
(prefix, suffixes) prompts; a stack served step by step needs something else:

* every attention layer owns pools ``[pages, page_size, width]``: keys (already normed / rotated) and
  values, or one pool of latent rows from which keys and values are made; a layer may read another
  layer's pools instead of owning any.  A request holds a list of page numbers, the same in every
  layer's pool, so one page table serves all layers.  Token at position p of a request sits in row
  ``p % page_size`` of page ``table[p // page_size]``;
* an attention layer that sees the tokens before its window as blocks of P positions owns block pools
  besides, ``[block pages, page_size, width]``: the mean key and the mean value of every complete block.
  A request's blocks have pages of their own (one list per P, whichever layers use it): block b sits in
  row ``b % page_size`` of block page ``block_table[P][b // page_size]``.  They are kept for as long as the
  request lives, also when the pages of the tokens they stand for have been given back;
* every recurrent layer owns ``[slots, ...]`` fp32 tensors: the recurrence's state and the last
  ``taps - 1`` inputs of its short convolution.  A request holds one slot number, the same in every
  layer.  A request that starts at position 0 never reads its slot (the kernels start from zeros),
  so a slot or page that is handed out again needs no clearing;
* a stack whose embedding looks at the token before has each request remember its last token;
* attention that only looks inside the current chunk of the sequence (or a window) never reads
  older keys again: :meth:`trim` gives pages wholly behind every layer's horizon back to the pool
  (never the pages of the first tokens that a window keeps for good).

Pools grow by doubling when they run out, so the sizes given at construction are hints.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence, Tuple

import numpy as np
import torch

PAGE_SIZE = 16


class _Request:
    __slots__ = ("slot", "pages", "length", "first_page", "block_pages", "last_token")

    def __init__(self, slot: int):
        self.slot = slot
        self.pages: List[int] = []     # page numbers from logical page ``first_page`` on (-1: given back)
        self.length = 0                # tokens stored so far
        self.first_page = 0
        self.last_token = -1           # (kept when the family's embedding reads the token before: ``prev_token``)
        self.block_pages: Dict[int, List[int]] = {}      # block length P -> pages of the request's blocks


class SequenceStateCache:
    def __init__(self, cfg, device, dtype: torch.dtype, max_tokens: int = 4096, max_seqs: int = 8,
                 page_size: int = PAGE_SIZE):
        self.cfg, self.dev, self.dtype, self.page_size = cfg, torch.device(device), dtype, int(page_size)
        # what the model family keeps per request (models.hybrid_family(cfg).state_spec):
        #   paged    layer -> {pool: row width}: pools [pages, page_size, width] of the GEMM type
        #   alias    layer -> the layer whose pools it reads (a layer that shares another's keys)
        #   blocks   layer -> (P, {pool: row width}): pools with one row per complete block of P positions
        #   slots    layer -> {tensor: shape}: fp32 [slots, *shape]
        #   horizons (kind, size, keep_first) of every layer that reads pages: "chunk": the keys of the
        #            current chunk of ``size`` positions; "window": the last ``size`` positions, and for
        #            good the first ``keep_first`` of the sequence
        #   prev_token  whether the embedding of a token reads the one before it
        from ..models import hybrid_family
        spec = hybrid_family(cfg).state_spec(cfg)
        self.attn: Dict[str, dict] = dict(spec["paged"])
        self.alias: Dict[str, str] = dict(spec.get("alias", {}))
        self.blocks: Dict[str, tuple] = {k: (int(P), dict(w)) for k, (P, w) in spec.get("blocks", {}).items()}
        self.block_sizes = sorted({P for P, _ in self.blocks.values()})
        self.rec: Dict[str, dict] = dict(spec["slots"])
        self.horizons = list(spec["horizons"])
        self.prev_token = bool(spec.get("prev_token", False))
        self.keep_pages = max([-(-int(k) // self.page_size) for _, _, k in self.horizons] + [0])
        self._kv: Dict[str, Dict[str, torch.Tensor]] = {}
        self._rec: Dict[str, Dict[str, torch.Tensor]] = {}
        self._blk: Dict[str, Dict[str, torch.Tensor]] = {}
        self.n_block_pages = {P: 0 for P in self.block_sizes}
        self.free_block_pages: Dict[int, List[int]] = {P: [] for P in self.block_sizes}
        self.block_pages_reused = 0
        self._ever_block_pages = {P: set() for P in self.block_sizes}
        self.n_pages = self.n_slots = 0
        self.free_pages: List[int] = []
        self.free_slots: List[int] = []
        self.requests: Dict[object, _Request] = {}
        self.pages_reused = self.slots_reused = self.pages_trimmed = 0
        self.generation = 0            # bumped when a pool is reallocated (captured graphs hold the old addresses)
        self._ever_pages, self._ever_slots = set(), set()
        self._grow_pages(max(2, -(-int(max_tokens) // self.page_size) + int(max_seqs)))
        self._grow_slots(max(1, int(max_seqs)))
        for P in self.block_sizes:
            self._grow_block_pages(P, max(1, int(max_tokens) // (P * self.page_size) + int(max_seqs)))

    # ------------------------------------------------------------------ pools
    def _grow_pages(self, n: int) -> None:
        if n <= self.n_pages:
            return
        for name, widths in self.attn.items():
            new = {k: torch.empty(n, self.page_size, w, dtype=self.dtype, device=self.dev) for k, w in widths.items()}
            if name in self._kv:
                for k in new:
                    new[k][:self.n_pages].copy_(self._kv[name][k])
            self._kv[name] = new
        self.free_pages = list(range(n - 1, self.n_pages - 1, -1)) + self.free_pages
        self.n_pages = n
        self.generation += 1

    def _grow_block_pages(self, P: int, n: int) -> None:
        old = self.n_block_pages[P]
        if n <= old:
            return
        for name, (size, widths) in self.blocks.items():
            if size != P:
                continue
            new = {k: torch.empty(n, self.page_size, w, dtype=self.dtype, device=self.dev) for k, w in widths.items()}
            if name in self._blk:
                for k in new:
                    new[k][:old].copy_(self._blk[name][k])
            self._blk[name] = new
        self.free_block_pages[P] = list(range(n - 1, old - 1, -1)) + self.free_block_pages[P]
        self.n_block_pages[P] = n
        self.generation += 1

    def _grow_slots(self, n: int) -> None:
        if n <= self.n_slots:
            return
        for name, r in self.rec.items():
            new = {k: torch.zeros((n,) + tuple(shape), dtype=torch.float32, device=self.dev) for k, shape in r.items()}
            if name in self._rec:
                for k in new:
                    new[k][:self.n_slots].copy_(self._rec[name][k])
            self._rec[name] = new
        self.free_slots = list(range(n - 1, self.n_slots - 1, -1)) + self.free_slots
        self.n_slots = n
        self.generation += 1

    def pools(self, layer: str) -> Dict[str, torch.Tensor]:
        """The page pools layer ``layer`` reads and writes (its own, or those of the layer it shares)."""
        return self._kv[self.alias.get(layer, layer)]

    def kv(self, layer: str) -> Tuple[torch.Tensor, torch.Tensor]:
        p = self.pools(layer)
        return p["k"], p["v"]

    def block_pools(self, layer: str, meta: dict) -> tuple:
        """(block keys, block values, the step's block page table, P) of an attention layer with pooled blocks."""
        P = self.blocks[layer][0]
        p = self._blk[layer]
        return p["k"], p["v"], meta[f"block_table_{P}"], P

    def recurrent(self, layer: str) -> Dict[str, torch.Tensor]:
        return self._rec[layer]

    def nbytes(self) -> int:
        n = sum(t.numel() * t.element_size() for pools in (self._kv, self._blk) for p in pools.values() for t in p.values())
        return n + sum(t.numel() * 4 for r in self._rec.values() for t in r.values())

    # --------------------------------------------------------------- requests
    def length(self, rid) -> int:
        r = self.requests.get(rid)
        return r.length if r is not None else 0

    def extend(self, rid, n_tokens: int) -> Tuple[int, int]:
        """Room for ``n_tokens`` more tokens of request ``rid`` (admitted at its first call) ->
        (position of the first of them, the request's state slot)."""
        r = self.requests.get(rid)
        if r is None:
            if not self.free_slots:
                self._grow_slots(2 * self.n_slots)
            s = self.free_slots.pop()
            self.slots_reused += s in self._ever_slots
            self._ever_slots.add(s)
            r = self.requests[rid] = _Request(s)
        pos0 = r.length
        need = -(-(pos0 + n_tokens) // self.page_size) - r.first_page
        while len(r.pages) < need:
            if not self.free_pages:
                self._grow_pages(2 * self.n_pages)
            p = self.free_pages.pop()
            self.pages_reused += p in self._ever_pages
            self._ever_pages.add(p)
            r.pages.append(p)
        for P in self.block_sizes:
            mine, free = r.block_pages.setdefault(P, []), self.free_block_pages
            need = -(-((pos0 + n_tokens) // P) // self.page_size)
            while len(mine) < need:
                if not free[P]:
                    self._grow_block_pages(P, 2 * self.n_block_pages[P])
                p = free[P].pop()
                self.block_pages_reused += p in self._ever_block_pages[P]
                self._ever_block_pages[P].add(p)
                mine.append(p)
        r.length = pos0 + n_tokens
        return pos0, r.slot

    def advance_token(self, rid, last: int) -> int:
        """The token before the request's rows of this step (-1: none); ``last``, their last one, takes its place."""
        r = self.requests[rid]
        prev, r.last_token = r.last_token, int(last)
        return prev

    def horizon(self, next_pos: int) -> int:
        """First position past the kept first tokens that any layer can still read once the token at
        ``next_pos`` runs."""
        lo = next_pos
        for kind, size, _ in self.horizons:
            lo = min(lo, (next_pos // size) * size if kind == "chunk" else max(0, next_pos - size + 1))
        return lo

    def trim(self, rid) -> int:
        """Give back the pages of ``rid`` that lie wholly behind every layer's horizon (and hold none of
        the first tokens a window keeps)."""
        r = self.requests.get(rid)
        if r is None or not self.horizons:
            return 0
        keep_from = self.horizon(r.length) // self.page_size
        n = 0
        for lp in range(max(r.first_page, self.keep_pages), min(keep_from, r.first_page + len(r.pages))):
            i = lp - r.first_page
            if r.pages[i] >= 0:
                self.free_pages.append(r.pages[i])
                r.pages[i] = -1
                n += 1
        self.pages_trimmed += n
        return n

    def release(self, rid) -> None:
        r = self.requests.pop(rid, None)
        if r is None:
            return
        self.free_pages += [p for p in r.pages if p >= 0]
        for P, pages in r.block_pages.items():
            self.free_block_pages[P] += pages
        self.free_slots.append(r.slot)

    def page_table(self, rids: Sequence) -> np.ndarray:
        """[len(rids), widest] int32 page numbers by logical page (-1: none)."""
        width = max([self.requests[i].first_page + len(self.requests[i].pages) for i in rids] + [1])
        t = np.full((len(rids), width), -1, dtype=np.int32)
        for j, i in enumerate(rids):
            r = self.requests[i]
            t[j, r.first_page:r.first_page + len(r.pages)] = r.pages
        return t

    def block_table(self, rids: Sequence, P: int) -> np.ndarray:
        """[len(rids), widest] int32 pages of the requests' blocks of P positions (-1: none)."""
        width = max([len(self.requests[i].block_pages.get(P, ())) for i in rids] + [1])
        t = np.full((len(rids), width), -1, dtype=np.int32)
        for j, i in enumerate(rids):
            pages = self.requests[i].block_pages.get(P, ())
            t[j, :len(pages)] = pages
        return t

    def live_tokens(self) -> int:
        return sum(r.length for r in self.requests.values())
