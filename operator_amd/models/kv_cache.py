"""Paged KV cache (SURVEY.md §2.4 N10/N12, §7.1 runtime/kvcache).

Layout per layer: K and V tensors [pages, Hkv_local, page_size, D] (bf16) —
a kv-head's tokens of one page are contiguous, which is what the decode
attention kernel streams (4 tokens = 1 KiB per wave load). All layers live in
two big allocations [L, pages, Hkv, P, D] sized up front from the HBM budget
(288 GB/GPU: for Llama-3-8B at 128 KiB/token, ~1.5M tokens fit beside the weights).

Page bookkeeping (free list, per-sequence page tables) is host-side and
O(pages) per request; block tables are uploaded as int32 rows.

``dtype=torch.float8_e4m3fn`` keeps K and V as OCP e4m3 with per-tensor scales
(``k_scale`` / ``v_scale``, stored value = x / scale): half the bytes per token,
so twice the tokens per GB and half the HBM traffic of decode attention, at
fp8 precision for the cached keys and values (queries and all compute stay
bf16 / fp32). Not the default.

``shapes`` gives every layer its own (kv heads, key size, value size): one K and one V
tensor per layer instead of the two stacked ones. How a layer arranges a page's bytes is its
kernels' business (attn_decode.hip's K tiles, qkv_heads.hip's K / V tiles). A layer that keeps
latent rows has one head and no values; one that reads another layer's rows has no heads.

``page_rows`` adds per layer a few rows of recurrent state to every page (``state``): the last
projections a short convolution asks for belong to the page of their tokens, so they are
allocated, shared with a common prefix and freed with it.
"""
from __future__ import annotations

import threading

import torch


class PageAllocator:
    """LIFO free list of page ids (recently freed pages are reused first: warm in L2/MALL)."""

    def __init__(self, num_pages: int):
        self.num_pages = num_pages
        self._free = list(range(num_pages - 1, -1, -1))
        self._lock = threading.Lock()

    @property
    def free(self) -> int:
        return len(self._free)

    def alloc(self, n: int) -> list[int]:
        with self._lock:
            if n > len(self._free):
                raise MemoryError(f"KV cache exhausted: need {n} pages, {len(self._free)} free")
            out = self._free[-n:][::-1] if n else []
            del self._free[len(self._free) - n:]
            return out

    def release(self, pages: list[int]) -> None:
        with self._lock:
            self._free.extend(reversed(pages))


class PagedKVCache:
    def __init__(self, layers: int, num_pages: int, kv_heads: int, head_dim: int, page_size: int = 64,
                 device: str | torch.device = "cuda", dtype: torch.dtype = torch.bfloat16,
                 k_scale: float = 1.0, v_scale: float = 1.0, shapes: list[tuple[int, int, int]] | None = None,
                 page_rows: list[tuple[int, int] | None] = ()):
        if page_size & (page_size - 1):
            raise ValueError("page_size must be a power of two")
        if k_scale <= 0 or v_scale <= 0:
            raise ValueError("KV scales must be positive")
        self.dtype, self.k_scale, self.v_scale = dtype, float(k_scale), float(v_scale)
        self.layers, self.num_pages, self.kv_heads, self.head_dim, self.page_size = (
            layers, num_pages, kv_heads, head_dim, page_size)
        if shapes is None:
            shape = (layers, num_pages, kv_heads, page_size, head_dim)
            self.k = torch.zeros(shape, dtype=dtype, device=device)
            self.v = torch.zeros(shape, dtype=dtype, device=device)
        else:
            new = lambda h, d: torch.zeros(num_pages, h, page_size, d, dtype=dtype, device=device)  # noqa: E731
            self.k = [new(h, dk) for h, dk, _ in shapes]
            self.v = [new(h, dv) for h, _, dv in shapes]
        self.state = [None if r is None else torch.zeros(num_pages, *r, dtype=dtype, device=device) for r in page_rows]
        self.allocator = PageAllocator(num_pages)

    @classmethod
    def for_model(cls, model, num_pages: int, page_size: int = 64, dtype: torch.dtype | None = None, k_scale: float = 1.0,
                  v_scale: float = 1.0) -> "PagedKVCache":
        """The cache ``model`` needs (its ``kv_shapes``), in its compute dtype unless given."""
        shapes = model.kv_shapes()
        h, dk, dv = shapes[0]
        rows = model.page_rows()
        if any(r is not None and r[0] > page_size for r in rows):
            raise ValueError(f"pages of {page_size} tokens cannot hold the state rows of {rows}")
        alike = dk == dv and all(s == shapes[0] for s in shapes)
        return cls(len(shapes), num_pages, h, dk, page_size, device=model.device, dtype=dtype or model.dtype,
                   k_scale=k_scale, v_scale=v_scale, shapes=None if alike else shapes, page_rows=rows)

    @staticmethod
    def pages_for_shapes(budget_bytes: int, shapes: list[tuple[int, int, int]], page_size: int, dtype_bytes: int = 2,
                         page_rows: list[tuple[int, int] | None] = ()) -> int:
        per_page = (sum(h * (dk + dv) for h, dk, dv in shapes) * page_size + sum(r * c for r, c in filter(None, page_rows))) * dtype_bytes
        return max(1, int(budget_bytes // per_page))

    @staticmethod
    def pages_for_budget(budget_bytes: int, layers: int, kv_heads: int, head_dim: int, page_size: int,
                         dtype_bytes: int = 2) -> int:
        per_page = 2 * layers * kv_heads * page_size * head_dim * dtype_bytes
        return max(1, int(budget_bytes // per_page))

    def pages_needed(self, tokens: int) -> int:
        return (tokens + self.page_size - 1) // self.page_size

    def layer(self, i: int) -> tuple[torch.Tensor, torch.Tensor]:
        return self.k[i], self.v[i]

    def slots_for(self, pages: list[int], start: int, n: int) -> list[int]:
        P = self.page_size
        return [pages[(start + j) // P] * P + (start + j) % P for j in range(n)]
