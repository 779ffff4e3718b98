"""Paged storage of latent attention: one vector per token and layer, of a width that may differ between layers.

The bookkeeping is PageAllocator's (64-token pages, reference counts, free list; one page id names the same slice of every layer's slab), the
slabs are this class's own: layer i holds [num_pages, 64, row_elems[i]] instead of a key block and a value block."""
from __future__ import annotations

import torch

from . import BaseCache
from .paged import TOKEN_CAPACITY_PER_PAGE, PageAllocator, PagedKVCache, PagedSequence


class LatentPageAllocator(PageAllocator):
    def __init__(self, num_pages: int, row_elems: list[int], dtype: torch.dtype = torch.bfloat16, device: torch.device | str | None = None):
        """row_elems: stored numbers per token, layer by layer (the latent's width, padded as the kernels want it)."""
        super().__init__(num_pages, 1, max([*row_elems, 1]), num_layers=len(row_elems))  # the native pool keeps the ids; it never touches pages
        self.dtype, self.row_elems = dtype, list(row_elems)
        self.slabs = None
        if device is not None:
            self.slabs = [torch.zeros(num_pages, TOKEN_CAPACITY_PER_PAGE, n, dtype=dtype, device=device) for n in row_elems]
        self.page_bytes = TOKEN_CAPACITY_PER_PAGE * sum(row_elems) * dtype.itemsize  # of all layers together

    @property
    def device(self) -> torch.device | None:
        return self.slabs[0].device if self.slabs else None

    def copy_page(self, src: int, dst: int) -> None:
        for s in self.slabs:
            s[dst] = s[src]


class SavedLatentCache(BaseCache):
    """One layer's latents as a file holds them ([1, 1, tokens, width]); a model copies them into its pages before it runs (adopt_cache)."""

    def __init__(self):
        self.rows: torch.Tensor | None = None
        self.offset = 0
        self.step = TOKEN_CAPACITY_PER_PAGE

    @property
    def state(self):
        return self.rows, None

    @state.setter
    def state(self, v):
        self.rows = v[0]
        self.offset = 0 if self.rows is None else self.rows.shape[2]

    def reuse(self, new_prompt_length: int, common_prefix_length: int) -> None:
        self.offset = min(self.offset, common_prefix_length)

    def is_trimmable(self) -> bool:
        return True

    def trim(self, n: int) -> int:
        n = min(self.offset, n)
        self.offset -= n
        return n

    def update_and_fetch(self, keys, values):
        raise NotImplementedError("saved latents are read-only; a model adopts them into its pages")

    def to_quantized(self, group_size: int = 64, bits: int = 4):
        return self


class PagedLatentCache(PagedKVCache):
    """Per-layer view of a PagedSequence over a LatentPageAllocator; reuse, trim and offset are the paged cache's."""

    def _rows(self, which: int) -> torch.Tensor:
        seq, a = self.page_manager, self.page_manager.allocator
        slab = a.slabs[self.layer]
        rows = slab[torch.tensor(seq.pages, dtype=torch.long, device=slab.device)] if seq.pages else slab[:0]
        return rows.reshape(-1, slab.shape[-1])[:seq.offset].reshape(1, 1, seq.offset, -1).contiguous()

    @property
    def state(self):
        return self._rows(0), None

    @state.setter
    def state(self, v):
        rows = v[0]
        seq, a = self.page_manager, self.page_manager.allocator
        n = rows.shape[2]
        if self.layer == 0 or seq.offset != n:
            seq.truncate(0)
            seq.reserve(n)
            seq.offset = n
            seq._mark_tokens()
        slab = a.slabs[self.layer]
        for j, p in enumerate(seq.pages):
            part = rows[0, 0, j * TOKEN_CAPACITY_PER_PAGE:(j + 1) * TOKEN_CAPACITY_PER_PAGE]
            slab[p, :part.shape[0]] = part.to(device=slab.device, dtype=slab.dtype)

    def adopt(self, saved: SavedLatentCache) -> None:
        """Takes over what a file held."""
        self.state = (saved.rows[:, :, :saved.offset], None)


__all__ = ["LatentPageAllocator", "PagedLatentCache", "SavedLatentCache", "PagedSequence"]
