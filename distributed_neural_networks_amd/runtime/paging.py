"""Paged KV cache bookkeeping: pages, block tables and the batch of one step.

* ``PageTable`` — the allocator of a pool of ``PAGE``-key pages shared by every
  layer of every stage: a sequence takes a slot (a row of the block table) when
  it is admitted, pages as its length grows, and gives both back when it ends.
  Freed pages and slots are used again first, so the pool only has to hold what
  is live.
* ``StepBatch`` — the device-side description of one engine step: tokens of any
  number of sequences, prompt portions and single decoded tokens together.

The page pools themselves belong to the stages (``runtime/decoder.py``); a page
id addresses the same page in each of them.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional, Sequence

import numpy as np
import torch

from ..ops.decoder_ops import LATENT_ROWS, PAGE, chunk_tiles


class OutOfPages(RuntimeError):
    """The pool (or the slots) cannot hold what was asked for; nothing was taken."""


def pages_for(tokens: int) -> int:
    return -(-tokens // PAGE)


class PageTable:
    def __init__(self, num_pages: int, max_slots: int, pages_per_slot: Optional[int] = None):
        if num_pages < 1 or max_slots < 1:
            raise ValueError("PageTable: at least one page and one slot")
        self.num_pages, self.max_slots = num_pages, max_slots
        self.width = pages_per_slot or num_pages
        self.table = np.full((max_slots, self.width), -1, dtype=np.int32)
        self._free_pages = list(range(num_pages - 1, -1, -1))  # stacks: the last freed is used next
        self._free_slots = list(range(max_slots - 1, -1, -1))
        self._held: Dict[int, List[int]] = {}

    @property
    def free_pages(self) -> int:
        return len(self._free_pages)

    @property
    def free_slots(self) -> int:
        return len(self._free_slots)

    def admit(self) -> int:
        """A free slot (block-table row), without pages yet."""
        if not self._free_slots:
            raise OutOfPages(f"all {self.max_slots} sequence slots are in use")
        slot = self._free_slots.pop()
        self._held[slot] = []
        return slot

    def missing(self, slot: int, tokens: int) -> int:
        """Pages the slot still needs to hold ``tokens`` positions."""
        return max(0, pages_for(tokens) - len(self._held[slot]))

    def reserve(self, slot: int, tokens: int) -> None:
        """Pages for positions 0 .. tokens - 1 of the slot's sequence."""
        held, need = self._held[slot], self.missing(slot, tokens)
        if need > len(self._free_pages) or len(held) + need > self.width:
            raise OutOfPages(f"{tokens} tokens need {need} more pages, {len(self._free_pages)} of {self.num_pages} free"
                             f" (at most {self.width} per sequence)")
        for _ in range(need):
            p = self._free_pages.pop()
            self.table[slot, len(held)] = p
            held.append(p)

    def release(self, slot: int) -> None:
        held = self._held.pop(slot)
        self._free_pages.extend(reversed(held))
        self.table[slot, :] = -1
        self._free_slots.append(slot)


@dataclass
class StepBatch:
    """One step's rows on the device.  ``chunks``: (first row, tokens, slot) of
    the sequences that bring two tokens or more; ``dec_rows``: rows of the
    sequences that bring one; ``ent``: {first row, tokens, slot, 0} of all of
    them, the chunks first; ``start`` / ``last``: per row, the first and last row
    of its sequence; ``max_len``: the longest sequence after the step.
    ``tiles``: attention workgroups by key (``tile_lists``)."""
    M: int
    pos: torch.Tensor
    slots: torch.Tensor
    table: torch.Tensor
    dec_rows: Optional[torch.Tensor]
    n_dec: int
    chunks: Sequence[tuple]
    max_len: int
    ent: torch.Tensor
    start: torch.Tensor
    last: torch.Tensor
    ids: Optional[torch.Tensor] = None
    want: Optional[torch.Tensor] = None
    n_want: int = 0
    tiles: Optional[Dict[object, torch.Tensor]] = None


KEY_ROWS = 1 << 15    # most keys of a step that are projected to heads
KEY_TOKENS = 32       # fewest tokens of a portion that does so


@dataclass(frozen=True)
class LatentHeads:
    """Attention of ``heads`` heads over one latent cache, as an entry of a
    stage's ``groups`` (an int there: query heads per KV head).  ``latent``,
    ``dim``, ``vdim``: padded columns of a latent, of a head's unrotated key and
    of its value; ``by_keys``: portions may be scored over keys."""
    heads: int
    latent: int = 128
    dim: int = 64
    vdim: int = 64
    by_keys: bool = False

    @property
    def rows(self) -> int:
        """Packed rows of a single token's tile."""
        return LATENT_ROWS[0] if self.heads <= LATENT_ROWS[0] else LATENT_ROWS[1]

    @property
    def per_token(self) -> int:
        return -(-self.heads // self.rows)

    def over_keys(self, n: int, p0: int) -> bool:
        """Is a portion of ``n`` tokens from position ``p0`` on cheaper over keys?
        What its scores save, against the projection of the keys before it."""
        per_key = self.latent * (self.dim + self.vdim)
        return self.by_keys and n >= KEY_TOKENS and n * (p0 + n / 2) * (2 * self.latent - self.dim - self.vdim) > p0 * per_key


def tile_lists(groups: Sequence, chunks: Sequence[tuple], ones: Sequence[tuple],
               starts: Optional[Sequence[int]] = None) -> Dict[object, list]:
    """Workgroups of the attention launches of a step.  ``chunks`` / ``ones``:
    (first row, tokens, slot) of the sequences that bring several tokens / one;
    ``starts``: first positions of the chunks, where known.  Key ``g`` (query
    heads per KV head): prefill tiles; for a ``LatentHeads``: ``(g, "chunks")`` and
    ``(g, "ones")``, tiles of either kind of sequence over latents; ``(g, "keys")``,
    tiles over keys, with the pages to gather in ``(g, "pages")``."""
    out: Dict[object, list] = {}
    for g in groups:
        if not isinstance(g, LatentHeads):
            out[g] = [t for c in chunks for t in chunk_tiles(*c, g)]
            continue
        over, keys, pages, rows = [], [], [], 0
        for i, (row, n, slot) in enumerate(chunks):
            blocks = 0 if starts is None else pages_for(starts[i] + n)
            if blocks and g.over_keys(n, starts[i]) and rows + blocks * PAGE <= KEY_ROWS:
                keys += chunk_tiles(row, n, rows, 1)
                pages += [(rows + b * PAGE, slot, b, 0) for b in range(blocks)]
                rows += blocks * PAGE
            else:
                over += chunk_tiles(row, n, slot, g.heads, LATENT_ROWS[1])
        out[g, "chunks"], out[g, "keys"], out[g, "pages"] = over, keys, pages
        out[g, "ones"] = [t for c in ones for t in chunk_tiles(*c, g.heads, g.rows)]
    return {k: v for k, v in out.items() if v}


def build_batch(entries: Sequence[tuple], table: np.ndarray, groups: Sequence[int], device) -> StepBatch:
    """``entries``: (token ids, first position, slot, wanted places) per
    sequence.  ``groups``: the kinds of attention of the model's layers
    (``tile_lists``).  Everything travels in one host-to-device copy."""
    ids, pos, slots, dec, want, chunks, starts, start, last = [], [], [], [], [], [], [], [], []
    for toks, p0, slot, places in entries:
        n, row = len(toks), len(ids)
        if n == 0:
            raise ValueError("a step entry brings at least one token")
        want += [row + w for w in places]
        ids += toks
        pos += range(p0, p0 + n)
        slots += [slot] * n
        start += [row] * n
        last += [row + n - 1] * n
        if n == 1:
            dec.append(row)
        else:
            chunks.append((row, n, slot))
            starts.append(p0)
    tiles = tile_lists(groups, chunks, [(r, 1, slots[r]) for r in dec], starts)
    parts = [(k, np.array(t, dtype=np.int32).reshape(-1)) for k, t in tiles.items()]
    ent = [(r, n, slot, 0) for r, n, slot in chunks] + [(r, 1, slots[r], 0) for r in dec]
    parts += [("ent", np.array(ent, dtype=np.int32).reshape(-1)), ("start", np.array(start, dtype=np.int32)),
              ("last", np.array(last, dtype=np.int32)),
              ("ids", np.array(ids, dtype=np.int32)), ("pos", np.array(pos, dtype=np.int32)),
              ("slots", np.array(slots, dtype=np.int32)), ("dec", np.array(dec, dtype=np.int32)),
              ("want", np.array(want, dtype=np.int32)), ("table", table.reshape(-1))]
    off, total = {}, 0
    for name, a in parts:
        off[name] = total
        total += -(-a.size // 4) * 4  # 16-byte aligned starts
    host = np.zeros(total, dtype=np.int32)
    for name, a in parts:
        host[off[name]:off[name] + a.size] = a
    dev = torch.from_numpy(host).to(device)
    v = {name: dev[off[name]:off[name] + a.size] for name, a in parts}
    return StepBatch(M=len(ids), pos=v["pos"], slots=v["slots"], table=v["table"].view(table.shape),
                     dec_rows=v["dec"] if dec else None, n_dec=len(dec), chunks=chunks,
                     max_len=max(pos) + 1, ent=v["ent"].view(-1, 4), start=v["start"], last=v["last"], ids=v["ids"],
                     want=v["want"] if want else None, n_want=len(want), tiles={k: v[k].view(-1, 4) for k in tiles})
