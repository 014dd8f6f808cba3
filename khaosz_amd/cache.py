"""Sequences and what they hold: pages of the paged attention caches and slots of the recurrent states.

A sequence takes one slot when it is opened and pages as it grows; both go back when it is closed.  A slot or a page
needs no clearing: the kernels read no state of a sequence at position 0 and no page row that the sequence has not
written.  Where every layer of the model attends to a window only, pages that fell behind it go back while the
sequence runs.
"""
from __future__ import annotations

from typing import Any, Dict, List, Optional, Sequence

import numpy as np
import torch

from .seq_ops import Batch


class FreeList:
    """Numbers 0 .. n handed out and taken back, the lowest free one first."""

    def __init__(self, n: int, what: str):
        self._free, self._what = list(range(n - 1, -1, -1)), what

    def take(self) -> int:
        if not self._free:
            raise RuntimeError(f"no free {self._what}")
        return self._free.pop()

    def give(self, i: int) -> None:
        if i in self._free:
            raise ValueError(f"{self._what} {i} is free already")
        self._free.append(i)
        self._free.sort(reverse=True)

    def __len__(self) -> int:
        return len(self._free)


class _Live:
    __slots__ = ("slot", "length", "released")

    def __init__(self, slot: int):
        self.slot, self.length, self.released = slot, 0, 0


class SequenceCache:
    """Storage for at most ``max_seqs`` sequences that together hold at most ``max_tokens`` tokens."""

    def __init__(self, model: Any, max_tokens: int, max_seqs: int = 1, page: int = 64):
        if max_tokens < 1 or max_seqs < 1 or page < 1:
            raise ValueError("max_tokens, max_seqs and page must be positive")
        self.page, self.width = page, (max_tokens + page - 1) // page  # table entries per sequence
        self.window: Optional[int] = model.window
        n_pages = self.width + max_seqs - 1                            # every sequence's last page may be partly empty
        self.slots, self.pages = FreeList(max_seqs, "sequence slot"), FreeList(n_pages, "cache page")
        self.table = np.full((max_seqs, self.width), -1, np.int64)
        self.state = model.new_sequence_state(max_seqs, n_pages, page, self.width * page)
        self.live: Dict[int, _Live] = {}

    def open(self) -> int:
        """A new, empty sequence; returns its handle."""
        slot = self.slots.take()
        self.live[slot] = _Live(slot)
        return slot

    def close(self, handle: int) -> None:
        s = self.live.pop(handle)
        for i in range(self.width):
            self._release(s.slot, i)
        self.slots.give(s.slot)

    def length(self, handle: int) -> int:
        return self.live[handle].length

    def _release(self, slot: int, logical: int) -> None:
        if self.table[slot, logical] >= 0:
            self.pages.give(int(self.table[slot, logical]))
            self.table[slot, logical] = -1

    def reserve(self, handles: Sequence[int], n: int) -> None:
        """Pages for ``n`` more tokens of each sequence (their length does not change yet)."""
        for h in handles:
            s = self.live[h]
            need = (s.length + n + self.page - 1) // self.page
            if need > self.width:
                raise ValueError(f"a sequence of {s.length + n} tokens does not fit the cache of {self.width * self.page}")
            for i in range(s.length // self.page, need):
                if self.table[s.slot, i] < 0:
                    self.table[s.slot, i] = self.pages.take()

    def commit(self, handles: Sequence[int], n: int) -> None:
        """The ``n`` tokens of each sequence are in; pages behind every window go back."""
        for h in handles:
            s = self.live[h]
            s.length += n
            if self.window is not None:
                # the next token, at position length, still sees length - window + 1
                keep = max(s.length - self.window + 1, 0) // self.page
                for i in range(s.released, keep):
                    self._release(s.slot, i)
                s.released = max(s.released, keep)

    def pack(self, handles: Sequence[int], ids: Sequence[Sequence[int]], out: np.ndarray) -> None:
        """Token ids, page table rows, positions and slots of a step as int64 words (positions and slots as int32)."""
        B, S, P = len(handles), len(ids[0]), self.width
        out[:B * S] = np.asarray(ids, np.int64).reshape(-1)
        out[B * S:B * (S + P)] = self.table[[self.live[h].slot for h in handles]].reshape(-1)
        tail = out[B * (S + P):].view(np.int32)
        tail[:B] = [self.live[h].length for h in handles]
        tail[B:2 * B] = [self.live[h].slot for h in handles]

    def words(self, B: int, S: int) -> int:
        return B * (S + self.width + 1)

    def unpack(self, buf: torch.Tensor, B: int, S: int):
        """(ids [B, S], Batch) as views of a device copy of ``pack``'s words."""
        P = self.width
        tail = buf[B * (S + P):B * (S + P + 1)].view(torch.int32)
        return buf[:B * S].view(B, S), Batch(tail[:B], tail[B:], buf[B * S:B * (S + P)].view(B, P), B, S)
