"""What a layer-stack sequence holds when its layers differ: pages of keys and values where a layer caches tokens, and a slot of recurrent state.

The pages are LatentPageAllocator's (one page id names the same slice of every layer's slab; a layer that caches no tokens has an empty one), but they are in
the kernels' own order inside, so a page means something as a whole only.  A slot names one [floats] block in every recurrent layer's state tensor: taken with
a sequence's first page, given back with its last, never cleared -- a sequence's first token starts from zero whatever the slot holds.  A recurrent state
cannot go back: such a sequence is continued or started over."""
from __future__ import annotations

import torch

from .latent import LatentPageAllocator, PagedLatentCache, SavedLatentCache
from .paged import TOKEN_CAPACITY_PER_PAGE, PagedSequence


class StackPageAllocator(LatentPageAllocator):
    def __init__(self, num_pages: int, row_elems: list[int], state_floats: list[int], num_slots: int, dtype: torch.dtype = torch.bfloat16,
                 device: torch.device | str | None = None):
        """state_floats: fp32 numbers of recurrent state per sequence, layer by layer (0: none)."""
        super().__init__(num_pages, row_elems, dtype=dtype, device=device)
        self.state_floats, self.num_slots = list(state_floats), num_slots
        self._home = torch.device(device) if device is not None else None
        self.states = [torch.zeros(num_slots, n, dtype=torch.float32, device=device) if n and device is not None else None for n in state_floats]
        self._free_slots = list(range(num_slots - 1, -1, -1))

    @property
    def recurrent(self) -> bool:
        return any(self.state_floats)

    def take_slot(self) -> int:
        if not self._free_slots:
            raise RuntimeError(f"state slots exhausted ({self.num_slots} live sequences)")
        return self._free_slots.pop()

    def give_slot(self, slot: int) -> None:
        if slot in self._free_slots or not 0 <= slot < self.num_slots:
            raise ValueError(f"state slot {slot} is not in use")
        self._free_slots.append(slot)

    def num_free_slots(self) -> int:
        return len(self._free_slots)

    def copy_slot(self, src: int, dst: int) -> None:
        for s in self.states:
            if s is not None:
                s[dst] = s[src]


class StackSequence(PagedSequence):
    """A PagedSequence that also holds a state slot while it holds tokens."""

    slot: int | None = None

    def reserve(self, needed: int) -> None:
        fresh = self.allocator.recurrent and self.slot is None
        if fresh:
            self.slot = self.allocator.take_slot()
        try:
            super().reserve(needed)
        except RuntimeError:
            if fresh:
                self._drop_slot()
            raise

    def _drop_slot(self) -> None:
        if self.slot is not None:
            self.allocator.give_slot(self.slot)
            self.slot = None

    def keepable(self, length: int) -> int:
        """The longest prefix of `length` tokens that the sequence can be cut to."""
        return length if not self.allocator.recurrent or length == self.offset else 0

    def truncate(self, length: int) -> None:
        length = max(0, min(length, self.offset))
        if length and self.keepable(length) != length:
            raise ValueError(f"a recurrent sequence of {self.offset} tokens cannot be cut to {length}: its state is the last token's")
        super().truncate(length)
        if length == 0:
            self._drop_slot()

    def fork(self) -> "StackSequence":
        plain = super().fork()
        other = StackSequence(self.allocator, plain.max_blocks)
        other.table, other.pages, other.offset = plain.table, plain.pages, plain.offset
        plain.pages, plain.offset = [], 0
        if self.slot is not None:
            try:
                other.slot = self.allocator.take_slot()
            except RuntimeError:
                other.release()
                raise
            self.allocator.copy_slot(self.slot, other.slot)
        return other


class SavedStackCache(SavedLatentCache):
    """One layer's pages ([1, 1, whole pages of tokens, width]) and recurrent state as a file holds them."""

    def __init__(self):
        super().__init__()
        self.recurrent: torch.Tensor | None = None
        self.whole = 0

    @property
    def state(self):
        return self.rows, self.recurrent

    @state.setter
    def state(self, v):
        self.rows, self.recurrent = v

    @property
    def meta_state(self):
        return str(self.whole)

    @meta_state.setter
    def meta_state(self, v):
        self.whole = self.offset = int(v or 0)

    def to_quantized(self, group_size: int = 64, bits: int = 4):
        return self


class PagedStackCache(PagedLatentCache):
    """Per-layer view of a StackSequence."""

    def reusable(self, length: int) -> int:
        """How many of the first `length` tokens can be kept (all layers of a sequence agree)."""
        return self.page_manager.keepable(length)

    def is_trimmable(self) -> bool:
        return not self.page_manager.allocator.recurrent

    def trim(self, n: int) -> int:
        n = min(self.offset, n)
        if self.layer == 0 and n:
            self.page_manager.truncate(self.offset - n)
        return n

    @property
    def state(self):
        seq, a = self.page_manager, self.page_manager.allocator
        slab, states = a.slabs[self.layer], a.states[self.layer]
        rows = None
        if slab.shape[-1]:
            rows = slab[torch.tensor(seq.pages, dtype=torch.long, device=slab.device)].reshape(1, 1, len(seq.pages) * TOKEN_CAPACITY_PER_PAGE, -1)
        return rows, None if states is None or seq.slot is None else states[seq.slot].clone()

    @state.setter
    def state(self, v):
        raise NotImplementedError("a layer-stack cache is restored as a whole (adopt)")

    @property
    def meta_state(self):
        return str(self.offset)

    def adopt(self, saved: SavedStackCache) -> None:
        seq, a = self.page_manager, self.page_manager.allocator
        n = saved.offset
        if self.layer == 0:
            seq.truncate(0)
            if n:
                seq.reserve(n)
                seq.offset = n
                seq._mark_tokens()
        if not n:
            return
        slab, states = a.slabs[self.layer], a.states[self.layer]
        if slab.shape[-1]:
            pages = saved.rows.reshape(-1, TOKEN_CAPACITY_PER_PAGE, slab.shape[-1])[:len(seq.pages)]
            slab[torch.tensor(seq.pages, dtype=torch.long, device=slab.device)] = pages.to(device=slab.device, dtype=slab.dtype)
        if states is not None:
            states[seq.slot] = saved.recurrent.to(device=states.device)


__all__ = ["PagedStackCache", "SavedStackCache", "StackPageAllocator", "StackSequence"]
