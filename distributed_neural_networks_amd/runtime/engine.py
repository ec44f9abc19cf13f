"""Continuous batching over paged decoder stages on one GPU.

``Engine.step`` runs one batch of unequal sequences — portions of prompts beside
single decoded tokens — through the stages and returns the logits asked for;
what earlier steps left in the cache is used as it is.  ``Engine.generate`` is
the scheduler on top: first-come admission while slots and pages last, prompts
cut to a token budget per step, every running sequence one token per step,
sampling on the device.  A sequence's pages are reserved at admission for its
whole length, so a running sequence never waits for memory.

The fixed-shape microbatch schedule (``runtime/scheduler.py DecodeRing``, HIP
graphs, several ranks) drives the same stages through ``step``.
"""
from __future__ import annotations

from collections import deque
from dataclasses import dataclass, field
from typing import Dict, Hashable, List, Optional, Sequence

import torch

from .paging import OutOfPages, PageTable, build_batch, pages_for


@dataclass
class Entry:
    """One sequence's share of a step: its next tokens, and the places among
    them whose logits are wanted."""
    id: Hashable
    tokens: List[int]
    want: Sequence[int] = ()


@dataclass
class _Live:
    slot: int
    length: int = 0


@dataclass
class _Request:
    id: int
    prompt: List[int]
    steps: int
    fed: int = 0
    out: List[int] = field(default_factory=list)


class Engine:
    def __init__(self, stages: Sequence, num_pages: Optional[int] = None, max_slots: int = 8):
        self.stages = list(stages)
        if not (self.stages[0].first and self.stages[-1].last):
            raise ValueError("Engine: the stages of one whole model are needed")
        for s in self.stages:
            if not hasattr(s, "step_batch"):
                raise ValueError(f"model {s.model!r} has no paged step; use the decode ring")
        self.device = self.stages[0].device
        pages = min(s.num_pages for s in self.stages)
        if num_pages is not None and num_pages > pages:
            raise ValueError(f"Engine: {num_pages} pages asked for, the stages hold {pages}")
        slots = min((s.num_slots for s in self.stages if getattr(s, "recurrent", False)), default=max_slots)
        if max_slots > slots:
            raise ValueError(f"Engine: {max_slots} slots asked for, the stages hold the states of {slots} sequences")
        self.table = PageTable(num_pages or pages, max_slots)
        self.vocab = self.stages[0].V
        self.groups = sorted({g for s in self.stages for g in s.groups}, key=str)
        self.max_tokens = min(s.max_tokens for s in self.stages)
        self.live: Dict[Hashable, _Live] = {}
        self._pos: Optional[torch.Tensor] = None

    # ------------------------------------------------------------------ one step
    def step(self, entries: Sequence[Entry]) -> Optional[torch.Tensor]:
        """Logits (wanted rows, vocab) in the order of the entries and of their
        ``want``; None when nothing is wanted.  A sequence is admitted at its
        first entry; ``end`` gives back what it holds.  Nothing is changed when
        the step cannot run (``OutOfPages``, ``ValueError``)."""
        seen = set()
        for e in entries:
            if not e.tokens or e.id in seen:
                raise ValueError(f"step: entry {e.id!r} is empty or given twice")
            seen.add(e.id)
            if min(e.tokens) < 0 or max(e.tokens) >= self.vocab:
                raise ValueError(f"step: entry {e.id!r} has a token outside the vocabulary of {self.vocab}")
            if any(not 0 <= w < len(e.tokens) for w in e.want):
                raise ValueError(f"step: entry {e.id!r} wants a place outside its tokens")
        if not entries:
            return None
        if sum(len(e.tokens) for e in entries) > self.max_tokens:
            raise ValueError(f"step: more than {self.max_tokens} tokens")
        new = [e for e in entries if e.id not in self.live]
        need = sum(pages_for(len(e.tokens)) for e in new)
        need += sum(self.table.missing(lv.slot, lv.length + len(e.tokens)) for e in entries
                    for lv in [self.live.get(e.id)] if lv is not None)
        if len(new) > self.table.free_slots or need > self.table.free_pages:
            raise OutOfPages(f"step needs {len(new)} slots and {need} pages; {self.table.free_slots} and "
                             f"{self.table.free_pages} are free")
        rows = []
        for e in entries:
            lv = self.live.get(e.id)
            if lv is None:
                lv = self.live[e.id] = _Live(self.table.admit())
            self.table.reserve(lv.slot, lv.length + len(e.tokens))
            rows.append((list(e.tokens), lv.length, lv.slot, list(e.want)))
            lv.length += len(e.tokens)
        b = build_batch(rows, self.table.table, self.groups, self.device)
        x = None
        for s in self.stages:
            x = s.step_batch(b, x)
        self._pos = b.pos[b.want.long()].contiguous() if b.n_want else None
        return x

    def end(self, seq_id: Hashable) -> None:
        self.table.release(self.live.pop(seq_id).slot)

    # ------------------------------------------------------------------ generation
    def generate(self, prompts: Sequence[Sequence[int]], steps: int, budget: int = 0) -> List[List[int]]:
        """``steps`` tokens after every prompt (unequal lengths, any number of
        prompts).  ``budget``: tokens of one step (0: what the stages hold)."""
        budget = min(budget or self.max_tokens, self.max_tokens)
        if steps < 1 or any(len(p) == 0 for p in prompts):
            raise ValueError("generate: steps >= 1 and non-empty prompts")
        if self.live:
            raise ValueError("generate: the engine still holds sequences")
        for p in prompts:
            if pages_for(len(p) + steps) > self.table.num_pages:
                raise OutOfPages(f"a prompt of {len(p)} tokens and {steps} steps exceed the cache pool")
        queue = deque(_Request(i, list(p), steps) for i, p in enumerate(prompts))
        running: List[_Request] = []
        done: Dict[int, List[int]] = {}
        promised: Dict[int, int] = {}  # pages of running requests up to their full length
        while queue or running:
            entries, left = [], budget
            for r in running:  # decoding sequences first: one token each
                if r.fed >= len(r.prompt) and left > 0:
                    entries.append((r, [r.out[-1]]))
                    left -= 1
            for r in running:  # prompts under way
                if r.fed < len(r.prompt) and left > 0:
                    n = min(left, len(r.prompt) - r.fed)
                    entries.append((r, r.prompt[r.fed:r.fed + n]))
                    left -= n
            while queue and left > 0 and len(running) < self.table.max_slots:
                r = queue[0]
                need = pages_for(len(r.prompt) + steps)
                if sum(promised.values()) + need > self.table.num_pages:
                    break
                queue.popleft()
                promised[r.id] = need
                running.append(r)
                n = min(left, len(r.prompt))
                entries.append((r, r.prompt[:n]))
                left -= n
            batch, sampled = [], []
            for r, toks in entries:
                if r.fed < len(r.prompt):
                    r.fed += len(toks)
                want = [len(toks) - 1] if r.fed >= len(r.prompt) else []
                sampled += [r] if want else []
                batch.append(Entry(r.id, toks, want))
            logits = self.step(batch)
            if logits is None:
                continue
            for r, t in zip(sampled, self.stages[-1].sample(logits, self._pos).tolist()):
                r.out.append(t)
                if len(r.out) == steps:
                    self.end(r.id)
                    del promised[r.id]
                    running.remove(r)
                    done[r.id] = r.out
        return [done[i] for i in range(len(prompts))]
