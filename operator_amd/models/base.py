"""What the engine needs of a decoder model, and what its models share.

``LLMEngine`` drives any class with this surface: ``cfg`` (layers, max_position, eos_ids),
``device`` / ``dtype``, ``forward(ForwardBatch, PagedKVCache)``, ``sample``, the per-layer
cache shapes (``kv_shapes``, ``page_rows``) and the prefill attention's work granularity (``prefill_plan``).
"""
from __future__ import annotations

import dataclasses
import hashlib
from dataclasses import dataclass, field

import torch

from operator_amd import ops
from operator_amd.parallel.comm import Group


@dataclass
class ForwardBatch:
    """Flattened tokens of one engine step (prefill or decode, never mixed)."""
    input_ids: torch.Tensor            # [T] int64
    positions: torch.Tensor            # [T] int64
    slots: torch.Tensor                # [T] int64 (cache slot, -1 = do not write)
    is_prefill: bool
    logits_index: torch.Tensor | None  # [n_out] int64 rows to produce logits for (None = all)
    # prefill
    seq_lens: list[int] = field(default_factory=list)
    prefill_work: tuple | None = None
    # shared prompt prefix (LLMEngine prefix sharing): (pk, pv, seq_pfx, pfx_lens), pk / pv the
    # cached post-RoPE K/V per layer ([P, Hkv, D] each); sequence s's tokens follow pfx_lens[s] of them
    prefix: tuple | None = None
    kv_sink: object = None   # called (layer, k, v) with each prefill layer's K/V (prefix capture)
    # per sequence the page of the tokens before its first row, -1: none ([S] int32; state that
    # lives in the pages continues from there)
    prev_pages: torch.Tensor | None = None
    residual_sink: object = None   # called (layer, x [T, hidden] fp32) with the residual after each layer
    # decode
    block_tables: torch.Tensor | None = None   # [B, max_pages] int32
    context_lens: torch.Tensor | None = None   # [B] int32 (including the new token)
    num_splits: int = 1


def _seed_for(seed: int, name: str) -> int:
    return int.from_bytes(hashlib.sha256(f"{seed}:{name}".encode()).digest()[:8], "little") & ((1 << 63) - 1)


class DecoderModel:
    LAYER = None            # dataclass of one layer's tensors (fields: Tensor | None)
    LAYOUT_FUNCS: tuple[str, ...] = ()   # methods whose source text defines the weight layout (weight_cache)

    cfg = None
    device: torch.device
    dtype: torch.dtype
    tp: Group
    fp8 = False
    gu_block: int | None = None
    vocab_offset = 0
    hq = hkv = 1            # heads of this rank (the widest layer's), for launch heuristics
    split_tokens: int | None = None   # shortest piece decode attention cuts a context into (None: the default)

    # ------------------------------------------------------------------ engine surface
    def kv_shapes(self) -> list[tuple[int, int, int]]:
        """(kv heads, key size, value size) each layer keeps in the cache."""
        raise NotImplementedError

    def prefix_shapes(self) -> list[tuple[int, int, int]]:
        """(heads, key size, value size) of the rows each layer's prefill attention reads of a shared
        prompt prefix."""
        return self.kv_shapes()

    def page_rows(self) -> list[tuple[int, int] | None]:
        """(rows, columns) of recurrent state each layer keeps per cache page (None: none), for layers that
        need the last few tokens' projections; a page holds that of its own tokens."""
        return []

    def prefill_plan(self) -> tuple[int, int]:
        """(attention variant, query rows per work item) of the prefill work list."""
        raise NotImplementedError

    def prefix_ok(self) -> bool:
        """Whether the prefill attention can start from a shared prompt prefix."""
        return True

    def forward(self, fb: ForwardBatch, kv) -> torch.Tensor:
        raise NotImplementedError

    def init_random(self, seed: int = 0) -> "DecoderModel":
        raise NotImplementedError

    def load_checkpoint(self, path: str) -> "DecoderModel":
        """Weights of a local checkpoint directory (its config.json defines ``cfg``)."""
        raise NotImplementedError

    # ------------------------------------------------------------------ shared
    def _randn(self, seed: int, name: str, shape, std: float) -> torch.Tensor:
        g = torch.Generator(device=self.device)
        g.manual_seed(_seed_for(seed, name))
        t = torch.randn(shape, generator=g, device=self.device, dtype=self.dtype)
        return t.mul_(std)

    def weight_bytes(self) -> int:
        n = sum(t.numel() * t.element_size() for t in (self.embed, self.final_norm, self.lm_head))
        for lw in self.layers:
            n += sum(t.numel() * t.element_size() for f in dataclasses.fields(lw)
                     if (t := getattr(lw, f.name)) is not None)
        return n

    def sample(self, logits: torch.Tensor, temperature: torch.Tensor, seeds: torch.Tensor,
               positions: torch.Tensor) -> torch.Tensor:
        """Sample one token per row; under TP each rank samples its vocab shard and the
        global winner is the max perturbed value (ties -> smaller token id)."""
        if self.tp.world == 1:
            return ops.sample(logits, temperature, seeds, positions)
        n = logits.shape[0]
        val = torch.empty(n, dtype=torch.float32, device=logits.device)
        tok = ops.sample(logits, temperature, seeds, positions, col_offset=self.vocab_offset, out_val=val)
        pair = torch.stack([val, tok.to(torch.float32)], 1)             # exact for ids < 2^24
        allp = self.tp.all_gather_into(pair)                             # [W, n, 2]
        vals, toks = allp[..., 0], allp[..., 1]
        best = vals.max(0).values
        cand = torch.where(vals == best.unsqueeze(0), toks, torch.full_like(toks, float("inf")))
        return cand.min(0).values.to(torch.long)
