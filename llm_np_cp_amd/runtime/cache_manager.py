"""Paged cache and state-slot bookkeeping (host side).

A sequence holds one slot (its row in the block table and in every
recurrent layer's state) and as many pages as its tokens need.  All
paged layers share the block table: page n of a sequence is the same page
number in every layer's cache.  Nothing is cleared when pages or slots
change hands: attention reads only positions the sequence has written,
and a token at position 0 starts its recurrences from zero.
"""

from __future__ import annotations

from typing import List, Optional

import numpy as np


class CacheFull(RuntimeError):
    """No free page or slot; nothing was allocated."""


class Sequence:
    __slots__ = ("slot", "pages", "length")

    def __init__(self, slot: int):
        self.slot = slot
        self.pages: List[int] = []
        self.length = 0            # tokens written so far


class CacheManager:
    def __init__(self, pages: int, slots: int, page_size: int,
                 max_seq: Optional[int] = None):
        if pages < 1 or slots < 1 or page_size < 1:
            raise ValueError("cache needs at least one page and one slot")
        self.page_size = page_size
        self.num_pages = pages
        self.num_slots = slots
        width = pages if max_seq is None else -(-max_seq // page_size)
        self.table = np.zeros((slots, min(pages, width)), dtype=np.int32)
        self.version = 0           # bumped whenever the table changes
        self._pages = list(range(pages - 1, -1, -1))
        self._slots = list(range(slots - 1, -1, -1))
        self._live = set()

    @property
    def free_pages(self) -> int:
        return len(self._pages)

    @property
    def free_slots(self) -> int:
        return len(self._slots)

    def open(self) -> Sequence:
        if not self._slots:
            raise CacheFull(f"all {self.num_slots} sequence slots are taken")
        s = Sequence(self._slots.pop())
        self._live.add(s)
        return s

    def pages_for(self, tokens: int) -> int:
        return -(-tokens // self.page_size)

    def missing(self, seq: Sequence, tokens: int) -> int:
        """Pages seq still needs to hold `tokens` tokens."""
        return max(0, self.pages_for(tokens) - len(seq.pages))

    def reserve(self, seq: Sequence, tokens: int) -> None:
        """Give seq pages for `tokens` tokens in total."""
        if seq not in self._live:
            raise ValueError("sequence is closed")
        n = self.missing(seq, tokens)
        if n == 0:
            return
        if len(seq.pages) + n > self.table.shape[1]:
            raise ValueError(
                f"{tokens} tokens exceed the {self.table.shape[1]} pages of "
                f"{self.page_size} a sequence can hold")
        if n > len(self._pages):
            raise CacheFull(f"{n} more pages needed, {len(self._pages)} of "
                            f"{self.num_pages} free")
        for _ in range(n):
            page = self._pages.pop()
            self.table[seq.slot, len(seq.pages)] = page
            seq.pages.append(page)
        self.version += 1

    def close(self, seq: Sequence) -> None:
        if seq not in self._live:
            raise ValueError("sequence is closed")
        self._live.discard(seq)
        self._pages.extend(reversed(seq.pages))
        self._slots.append(seq.slot)
        seq.pages = []

    def close_all(self) -> None:
        for s in list(self._live):
            self.close(s)
