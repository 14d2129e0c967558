"""Trace replay: given token ids through a served model, step by step, logits out.

Every stdin line is one step as JSON:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

The entries of a step are one batch, either all new (their tokens are a prompt) or all going
on by one token. ``want`` are places among an entry's tokens whose logits are written, in
order, to OUT/<step>.f32 (little-endian fp32 [wanted, vocab]; no file when nothing is
wanted); requests in ``end`` give their cache pages back after the step. ``done <step>`` is
printed after each. The engine is the one the configuration serves with (``build_engine``):
its prefill packing, decode graphs, page tables and kernels.
"""
from __future__ import annotations

import json
import os
import sys

import torch

from operator_amd.config import Settings


class TraceReplay:
    def __init__(self, engine):
        self.engine = engine
        self.live: dict = {}

    def step(self, entries: list[dict], end: list) -> torch.Tensor | None:
        """Run one step; logits [wanted, vocab] (fp32) or None when nothing is wanted."""
        eng = self.engine
        new = [e["id"] not in self.live for e in entries]
        logits = None
        if entries and all(new):
            reqs, logits = eng.given_start([e["tokens"] for e in entries], [e.get("want", []) for e in entries])
            self.live.update((e["id"], r) for e, r in zip(entries, reqs))
        elif entries:
            if any(new) or any(len(e["tokens"]) != 1 for e in entries):
                raise ValueError("the entries of a step are all new or all go on by one token")
            out = eng.given_next([self.live[e["id"]] for e in entries], [e["tokens"][0] for e in entries])
            rows = [i for i, e in enumerate(entries) for _ in e.get("want", [])]
            logits = out[torch.tensor(rows, device=out.device)] if rows else None
        for rid in end:
            eng.given_end(self.live.pop(rid))
        return None if logits is None else logits.float()


def replay_engine(model_dir: str, dtype: str, max_tokens: int, s: Settings):
    """The serving engine of a checkpoint directory, its cache sized for ``max_tokens`` live
    tokens (each request may leave a page partly used)."""
    from operator_amd.engine.factory import build_engine

    e = s.engine
    e.model, e.model_path, e.dtype = os.path.basename(os.path.normpath(model_dir)), model_dir, dtype
    e.max_context = max(e.page_size, max_tokens)
    while -(-e.max_context // e.page_size) > 1024:   # page ids per sequence the decode attention holds
        e.page_size *= 2
    e.prefix_sharing = False   # every token's logits may be wanted, shared ones included
    return build_engine(s, kv_pages=-(-e.max_context // e.page_size) + min(max_tokens, 1024))


def replay(model_dir: str, dtype: str, out: str, max_tokens: int, s: Settings, stdin=None) -> int:
    torch.backends.cuda.matmul.allow_tf32 = False
    rp = TraceReplay(replay_engine(model_dir, dtype, max_tokens, s)[2])
    os.makedirs(out, exist_ok=True)
    for line in stdin or sys.stdin:
        if not line.strip():
            continue
        st = json.loads(line)
        logits = rp.step(st["entries"], st.get("end", []))
        if logits is not None:
            path = os.path.join(out, f"{st['step']}.f32")
            logits.cpu().contiguous().numpy().astype("<f4").tofile(path)
        print(f"done {st['step']}", flush=True)
    return 0
