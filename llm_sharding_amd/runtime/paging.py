"""Paged cache memory: a pool of fixed-size pages and one page table per cache slot.

The pool holds ``pages`` pages of ``page_tokens`` tokens each, whatever the number of slots and the
longest sequence: a slot takes pages as its sequence grows (:meth:`ensure`) and gives all of them
back at its end (:meth:`release`); the next sequence that needs one takes it, contents and all -
readers never look past a sequence's length. One table serves every layer of a stage (page p of
layer l is row p of that layer's cache tensor).

The tables live on the host (the truth) and on the device, where kernels and captured graphs read
them: entry -1 is "no page", which a kernel treats as an idle slot.
"""
from __future__ import annotations

import torch


class PagePool:
    def __init__(self, pages: int, slots: int, max_seq: int, page_tokens: int = 64, device="cpu"):
        if pages < 1 or slots < 1 or max_seq < 1:
            raise ValueError("a page pool needs pages, slots and a sequence length")
        self.pages, self.slots, self.page_tokens = int(pages), int(slots), int(page_tokens)
        self.max_pages = -(-int(max_seq) // page_tokens)
        self.free = list(range(self.pages - 1, -1, -1))  # a stack: the page given back last goes first
        self.held = [[] for _ in range(self.slots)]
        self.table = torch.full((self.slots, self.max_pages), -1, dtype=torch.int32, device=device)

    def pages_for(self, tokens: int) -> int:
        return -(-int(tokens) // self.page_tokens)

    def room_for(self, slot: int, tokens: int) -> bool:
        return self.pages_for(tokens) - len(self.held[slot]) <= len(self.free)

    def capacity(self, slot: int) -> int:
        """Tokens slot's pages hold."""
        return len(self.held[slot]) * self.page_tokens

    def ensure(self, slot: int, tokens: int) -> None:
        """Pages for the first ``tokens`` tokens of ``slot``."""
        have, need = len(self.held[slot]), self.pages_for(tokens)
        if need <= have:
            return
        if need > self.max_pages:
            raise ValueError(f"slot {slot}: {tokens} tokens exceed the longest sequence "
                             f"({self.max_pages * self.page_tokens})")
        if need - have > len(self.free):
            raise RuntimeError(f"slot {slot}: {need - have} cache pages needed, {len(self.free)} of {self.pages} free")
        new = [self.free.pop() for _ in range(need - have)]
        self.held[slot] += new
        self.table[slot, have:need] = torch.tensor(new, dtype=torch.int32).to(self.table.device)

    def release(self, slot: int) -> None:
        """Every page of ``slot`` back to the pool."""
        if self.held[slot]:
            self.free += reversed(self.held[slot])
            self.held[slot] = []
            self.table[slot].fill_(-1)


__all__ = ["PagePool"]
