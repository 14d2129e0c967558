"""Throughput of models at layer level: ``bench.py --model-speed``.

Each model is cut to a few layers (random weights) and driven through its engine's captured
graphs: prefill of packed equal prompts, decode steps of a batch at a given context. One
JSON line per case with the time, the rate and the roofline time of the same work (matrix
flops at the dense bf16 peak or the bytes a step must move at HBM peak, whichever is longer),
so models of one size compare by how far they are from their own bound.
"""
from __future__ import annotations

import gc
import json
from dataclasses import replace

import torch

from operator_amd.models.config import LatentSpec

PEAK_FLOPS, PEAK_BYTES = 2.5e15, 8.0e12
PREFILL = ((1, 1024), (8, 1024), (4, 4096))      # sequences, tokens each
DECODE = ((1, 1024), (64, 1024), (256, 1024), (64, 4096))   # rows, context


def cut(cfg, layers: int):
    """``cfg`` with its first ``layers`` layers."""
    if hasattr(cfg, "layer_specs"):
        return replace(cfg, layer_specs=cfg.layer_specs[:layers])
    return replace(cfg, layers=layers)


def _work(cfg, tokens: int, seqs: int, ctx: int, decode: bool) -> tuple[float, float]:
    """(matrix flops, bytes that must move) of one step: weights read once, keys and values (inside
    the window, or latent rows), fp32 residual streams where a model has them; only the experts in use."""
    def ff(h, f):
        return 3 * h * f

    h, flops, byts = cfg.hidden, 0.0, 0.0
    pairs = tokens * ctx if decode else tokens * (ctx + 1) / 2
    for i in range(cfg.layers):
        if cfg.arch == "relurax":
            m, f = cfg.layer_specs[i].mixer, cfg.layer_specs[i].mlp
            act = 0 if f is None else ff(h, f.ff)
            byts += 2 * 2 * tokens * h * 4
            if isinstance(m, LatentSpec):
                low = h * m.q_rank + m.q_rank * m.heads * (m.dim + m.rot_dim) + h * m.heads + m.heads * m.vdim * h
                low += h * (m.kv_rank + m.rot_dim) if m.kv_from < 0 else 0
                up = m.heads * (m.dim + m.vdim) * m.kv_rank
                per = m.heads * (2 * m.kv_rank + m.rot_dim if decode else m.dim + m.rot_dim + m.vdim)
                flops += 2 * tokens * (low + up + act) + 2 * pairs * per
                byts += 2 * (low + up + act) + 2 * (m.kv_rank + m.rot_dim) * (tokens * ctx if decode else tokens)
            else:
                proj = h * ((m.heads + m.kv_heads) * m.dim + m.heads) + h * m.heads * m.vdim
                w = min(m.window or ctx, ctx)
                seen = tokens * w if decode else tokens / ctx * (w * (w + 1) / 2 + (ctx - w) * w)
                flops += 2 * tokens * (proj + act) + 2 * seen * m.heads * (m.dim + m.vdim)
                byts += 2 * (proj + act) + 2 * m.kv_heads * (m.dim + m.vdim) * (tokens * w if decode else tokens)
            continue
        if cfg.arch == "sufolix":
            a, m = cfg.layer_specs[i].mixer, cfg.layer_specs[i].mlp
            heads, kv, dk, dv = a.heads, a.kv_heads, a.dim, a.vdim
            act = 0 if m is None else ff(h, m.ff) * (m.top if m.experts else 1) + (ff(h, m.shared_ff) if m.shared_ff else 0)
            used = 0 if m is None else ff(h, m.ff) * (min(m.experts, tokens * m.top) if m.experts else 1) + \
                (ff(h, m.shared_ff) if m.shared_ff else 0)
            byts += 2 * 2 * cfg.streams * tokens * h * 4
        else:
            heads, kv, dk, dv = cfg.heads, cfg.kv_heads, cfg.head_dim, cfg.head_dim
            act = used = ff(h, cfg.intermediate)
            byts += 2 * 2 * tokens * h * 2
        proj = h * ((heads + kv) * dk + kv * dv) + h * heads * dv
        flops += 2 * tokens * (proj + act) + 2 * pairs * heads * (dk + dv)
        byts += 2 * (proj + used) + 2 * kv * (dk + dv) * (tokens * ctx if decode else tokens)
    head = cfg.vocab_size * h
    return flops + 2 * seqs * head, byts + 2 * head


def _bound_ms(work) -> float:
    return max(work[0] / PEAK_FLOPS, work[1] / PEAK_BYTES) * 1e3


def _time(fn, iters: int) -> float:
    """Mean milliseconds of ``fn`` over ``iters`` back-to-back launches (best of 3)."""
    fn()
    torch.cuda.synchronize()
    best = float("inf")
    for _ in range(3):
        a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        a.record()
        for _ in range(iters):
            fn()
        b.record()
        b.synchronize()
        best = min(best, a.elapsed_time(b) / iters)
    return best


def run(names: list[str], layers: int = 4, prefill=PREFILL, decode=DECODE, emit=print) -> list[dict]:
    from operator_amd.engine.llm import GenRequest, LLMEngine
    from operator_amd.models.kv_cache import PagedKVCache
    from operator_amd.models.registry import build_model, load_config

    out = []
    for name in names:
        cfg = cut(load_config(name), layers)
        model = build_model(cfg, device="cuda").init_random(seed=1)
        P = 16
        need = max([b * (c // P + 2) for b, c in decode] + [b * (c // P + 1) for b, c in prefill])
        kv = PagedKVCache.for_model(model, need, P)
        eng = LLMEngine(model, kv, max_batch=256, max_prefill_tokens=max(b * c for b, c in prefill), max_context=8192,
                        prefix_sharing=False)

        def emit_case(kind, b, c, ms, tokens):
            bound = _bound_ms(_work(cfg, tokens, b, c, kind == "decode"))
            rec = {"model": name, "layers": cfg.layers, "phase": kind, "batch": b, "context": c, "ms": round(ms, 4),
                   "tokens_per_s": round(tokens / ms * 1e3), "bound_ms": round(bound, 4), "x_bound": round(ms / bound, 2)}
            out.append(rec)
            emit(json.dumps(rec))

        for b, c in prefill:
            reqs = [GenRequest(torch.randint(0, cfg.vocab_size, (c,)).tolist()) for _ in range(b)]
            for r in reqs:
                eng._reserve(r)
            p = eng._pack_prefill(reqs)
            eng.prefill_buckets = sorted({*eng.prefill_buckets, b * c})
            g = eng._prefill_graph(b * c)
            last = p["cu"][1:] - 1
            g.run(p["ids"], p["pos"], p["slots"], p["cu"], p["ws"], p["wq"], last, [0.0] * b, [0] * b, p["full"], p["skip"])
            emit_case("prefill", b, c, _time(g.graph.replay, 4), b * c)
            for r in reqs:
                eng.given_end(r)
        for b, c in decode:
            # rows with tokens (and sampling seeds) of their own: equal rows would share their experts
            reqs = [GenRequest([1] * (c - 1), output=[int(t)], temperature=1.0, seed=i)
                    for i, t in enumerate(torch.randint(0, cfg.vocab_size, (b,)))]
            for r in reqs:
                eng._reserve(r)
                r.pages = r.pages + kv.allocator.alloc(1)   # the steps below pass the page's end
            bp = eng._bucket(b)
            g = eng._graph(bp, eng._splits(c, bp))

            def steps():
                g.st.load(reqs, eng.max_pages)
                for _ in range(8):
                    g.graph.replay()

            emit_case("decode", b, c, _time(steps, 4) / 8, b)
            for r in reqs:
                eng.given_end(r)
        del eng, model, kv
        gc.collect()
        torch.cuda.empty_cache()
    return out
