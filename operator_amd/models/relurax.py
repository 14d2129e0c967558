"""Relurax decoder on the gfx950 kernels.

One fp32 residual stream with a norm before and after every sublayer, x += post(f(pre(x))). Per
layer (ops/decoder.py), with the stream step fused around every sublayer:

  window attention
    z      = h Win^T                             GEMM (q | k | gates; split-K slabs at decode)
    q,k,v,g = conv_heads(z)                      HIP  (short convolution, q/k norm, values = the
                                                       convolved keys, gate sigmoid, KV + state write)
    o      = g * attn(q, K, V, window)           HIP  (MFMA flash prefill | split-KV paged decode)
  latent attention (the cache keeps one row [c | rotated key part] per token)
    z      = h Win^T                             GEMM (query latent | latent row | gates)
    cq,row,g = latent_rows(z)                    HIP  (both norms, rotation, cache write, gate sigmoid)
    q      = rotate(cq Wuq^T)                    GEMM + HIP
    prefill: k, v = row Wk^T, row Wv^T           GEMM (Wk passes the rotated part through by an identity
             o = g * attn(q, k, v)               block), HIP
    decode:  q' = q_h Wuk_h, o' = g * attn(q', rows), o = o'_h Wuv_h^T    HIP, in the latent space
  y = o Wo^T, x += post(y), h = pre(x)           GEMM, HIP
  feed-forward: tanh-gelu gated (GEMM with fused epilogue), GEMM, and the same step
logits = norm(x) Wlm^T.

Weights are stored padded with zeros (models/padded.py). bf16 or fp32 (true 32-bit products)
throughout; residual, norms, rotation, gates' sigmoids, scores and softmax are fp32 in both.
"""
from __future__ import annotations

import math
from dataclasses import dataclass

import torch

from operator_amd import ops
from operator_amd.ops import decoder as dec
from operator_amd.parallel.comm import Group

from .base import ForwardBatch
from .config import LatentSpec, ReluraxConfig
from .kv_cache import PagedKVCache
from .padded import PaddedModel


@dataclass
class ReluraxLayer:
    """One layer's tensors (fp32 where small constants, the compute dtype for the products)."""
    win: torch.Tensor             # [ncol, ld]: q | k | gate rows, or query latent | latent | rotated part | gate rows
    wo: torch.Tensor              # [ld, ocol]
    norm1: torch.Tensor           # [ld] fp32
    norm1b: torch.Tensor
    qnorm: torch.Tensor           # [dk] of a head in the compute dtype, or [qp] of the query latent, fp32
    knorm: torch.Tensor | None = None   # [dk], or [rp] of the latent (None: it reads another layer's rows)
    conv: torch.Tensor | None = None    # [taps, (H + G) dk] in the compute dtype
    wuq: torch.Tensor | None = None     # latent: [H dk, qp]
    wk: torch.Tensor | None = None      # [H dk, ck] keys of all heads from a latent row
    wv: torch.Tensor | None = None      # [H dv, ck]
    wabs: torch.Tensor | None = None    # [H, rp, pad16(dim)] queries into the latent space
    wuv: torch.Tensor | None = None     # [H, dv, rp] values out of it
    norm2: torch.Tensor | None = None   # feed-forward (None: the layer has none)
    norm2b: torch.Tensor | None = None
    wgu: torch.Tensor | None = None     # [2 ff, ld], 64-row interleaved
    wd: torch.Tensor | None = None      # [ld, ff]


class ReluraxModel(PaddedModel):
    LAYER = ReluraxLayer
    LAYOUT_FUNCS = PaddedModel.LAYOUT_FUNCS + ("init_random", "_layer", "_attention", "_latent")

    def __init__(self, cfg: ReluraxConfig, device: str | torch.device = "cuda", tp: Group | None = None,
                 dtype: torch.dtype = torch.bfloat16, weight_dtype: str = "bfloat16"):
        super().__init__(cfg, device, tp, dtype, weight_dtype)
        self.shapes: list = []
        self.rot: list = []
        tabs: dict = {}
        for a in (sp.mixer for sp in cfg.layer_specs):
            if isinstance(a, LatentSpec):
                self.shapes.append(dec.LatentLayout(a.heads, a.dim, a.rot_dim, a.vdim, a.q_rank, a.kv_rank, a.kv_from < 0, cfg.rms_eps))
                key = (a.rot_base, a.rot_dim)
                if key not in tabs:
                    tabs[key] = dec.rotary_tables(cfg.max_position, a.rot_base, max(a.rot_dim, 2), device=self.device)
                self.rot.append(tabs[key])
            else:
                self.shapes.append(dec.HeadLayout(a.heads, a.kv_heads, a.dim, a.vdim, eps=cfg.rms_eps))
                self.rot.append(None)
        self.hq = max(L.heads for L in self.shapes)
        # decode workgroups per sequence of the layers that read whole contexts (chunks of 32 heads
        # over one latent row, or key/value heads): what the split count is chosen for
        full = [-(-L.heads // 32) for L in self.shapes if isinstance(L, dec.LatentLayout)]
        full += [L.kv_heads for L, sp in zip(self.shapes, cfg.layer_specs) if isinstance(L, dec.HeadLayout) and not sp.mixer.window]
        self.split_tokens = 128 if full else None   # latent rows are a few cache lines: short pieces pay
        self.hkv = min(full) if full else max(L.kv_heads for L in self.shapes)
        one = torch.ones(1, device=self.device)
        self.hc = dec.Stream(one, one.view(1, 1), one)   # a single residual stream

    # ------------------------------------------------------------------ engine surface
    def kv_shapes(self) -> list[tuple[int, int, int]]:
        return [(L.kv_heads, *L.pads) if isinstance(L, dec.HeadLayout) else (1 if L.own else 0, L.ck, 0) for L in self.shapes]

    def prefix_shapes(self) -> list[tuple[int, int, int]]:
        return [(L.kv_heads if isinstance(L, dec.HeadLayout) else L.heads, *L.pads) for L in self.shapes]

    def page_rows(self) -> list[tuple[int, int] | None]:
        return [(sp.mixer.conv - 1, (L.heads + L.kv_heads) * L.pads[0]) if isinstance(L, dec.HeadLayout) and sp.mixer.conv > 1 else None
                for L, sp in zip(self.shapes, self.cfg.layer_specs)]

    # ------------------------------------------------------------------ weights
    def _layer(self, i: int, get, has) -> ReluraxLayer:
        W, m, p = self.cfg.hidden, self.cfg.layer_specs[i].mlp, f"l{i}."
        norm = lambda n: self._padded(get(p + n, (W,)), self.ld)  # noqa: E731
        mix = self._latent if isinstance(self.shapes[i], dec.LatentLayout) else self._attention
        lw = ReluraxLayer(norm1=norm("norm1"), norm1b=norm("norm1b"), **mix(i, get, p + "mix."))
        if m is not None:
            lw.norm2, lw.norm2b = norm("norm2"), norm("norm2b")
            lw.wgu = self._gate_up(get(p + "mlp.gate", (m.ff, W)), get(p + "mlp.up", (m.ff, W)))
            lw.wd = self._down(get(p + "mlp.down", (W, m.ff)))
        return lw

    def _attention(self, i: int, get, p: str) -> dict:
        L, a, W = self.shapes[i], self.cfg.layer_specs[i].mixer, self.cfg.hidden
        (dk, dv), H, G, D = L.pads, L.heads, L.kv_heads, L.dim
        rows, at = [], 0
        conv = torch.zeros(a.conv, (H + G) * dk, dtype=self.dtype, device=self.device)
        for n, heads in (("q", H), ("k", G)):
            w, c = get(p + n, (heads * D, W)), get(p + n + ".conv", (heads * D, a.conv))
            for h in range(heads):
                rows.append((at, 0, w[h * D:(h + 1) * D]))
                conv[:, at:at + D] = c[h * D:(h + 1) * D].t()
                at += dk
        wo = get(p + "o", (W, H * D))
        return dict(win=self._put(dec.conv_ncol(L), self.ld, rows + [(at, 0, get(p + "g", (H, W)))]), conv=conv,
                    wo=self._put(self.ld, L.ocol, [(0, h * dv, wo[:, h * D:(h + 1) * D]) for h in range(H)]),
                    qnorm=self._padded(get(p + "q.norm", (D,)), dk).to(self.dtype), knorm=self._padded(get(p + "k.norm", (D,)), dk).to(self.dtype))

    def _latent(self, i: int, get, p: str) -> dict:
        L, W = self.shapes[i], self.cfg.hidden
        (dk, dv), H, D, R, V, C = L.pads, L.heads, L.dim, L.rot, L.vdim, L.kv_rank
        rows, at = [(0, 0, get(p + "dq", (L.q_rank, W)))], L.qp
        if L.own:
            w = get(p + "dkv", (C + R, W))
            rows += [(at, 0, w[:C]), (at + L.rp, 0, w[C:])]
            at += L.rp + L.rotp
        rows.append((at, 0, get(p + "g", (H, W))))
        uq, uk, uv = get(p + "uq", (H * (D + R), L.q_rank)), get(p + "uk", (H * D, C)), get(p + "uv", (H * V, C))
        wo = get(p + "o", (W, H * V))
        keys, values = [], []
        wabs = torch.zeros(H, L.rp, dec.pad_to(D, 16), dtype=self.dtype, device=self.device)
        wuv = torch.zeros(H, dv, L.rp, dtype=self.dtype, device=self.device)
        eye = torch.eye(R, dtype=self.dtype, device=self.device)
        for h in range(H):
            keys += [(h * dk, 0, uk[h * D:(h + 1) * D]), (h * dk + D, L.rp, eye)]
            values.append((h * dv, 0, uv[h * V:(h + 1) * V]))
            wabs[h, :C, :D] = uk[h * D:(h + 1) * D].t()
            wuv[h, :V, :C] = uv[h * V:(h + 1) * V]
        return dict(win=self._put(L.ncol, self.ld, rows), qnorm=self._padded(get(p + "dq.norm", (L.q_rank,)), L.qp),
                    knorm=self._padded(get(p + "dkv.norm", (C,)), L.rp) if L.own else None,
                    wuq=self._put(H * dk, L.qp, [(h * dk, 0, uq[h * (D + R):(h + 1) * (D + R)]) for h in range(H)]),
                    wk=self._put(H * dk, L.ck, keys), wv=self._put(H * dv, L.ck, values), wabs=wabs, wuv=wuv,
                    wo=self._put(self.ld, L.ocol, [(0, h * dv, wo[:, h * V:(h + 1) * V]) for h in range(H)]))

    def init_random(self, seed: int = 0) -> "ReluraxModel":
        """Random weights of the exact architecture with O(1) activations."""
        def get(name, shape):
            t = self._randn(seed, name, shape, 1.0)
            leaf = name.split(".")[-1]
            if leaf.startswith("norm"):
                return 1.0 + 0.1 * t
            if leaf == "conv":
                return t * (1.0 / math.sqrt(shape[-1]))
            return t if leaf == "embed" else t * (1.0 / math.sqrt(shape[-1]))

        return self._build(get, lambda name: True)

    # ------------------------------------------------------------------ forward
    def forward(self, fb: ForwardBatch, kv: PagedKVCache) -> torch.Tensor:
        """Run all layers; returns logits [n_out, vocab] for fb.logits_index rows."""
        c, one = self.cfg, self.hc.inp
        x, h = dec.stream_init(fb.input_ids, self.embed, 1.0, 1, c.hidden, one, self.layers[0].norm1, c.rms_eps)
        ws = None
        if fb.is_prefill:
            cu = None if fb.prefill_work is None else fb.prefill_work[0]
            edges = dec.SequenceEdges(cu, fb.seq_lens, fb.prev_pages)
        else:
            edges = dec.SequenceEdges(block_tables=fb.block_tables)
            if h.is_cuda:   # split-KV partials, shared by every layer
                ws = dec.attn_gd_workspace(h.shape[0], self.shapes, fb.num_splits, h.device)
        rows: dict = {}   # latent rows of this prefill, by the layer that keeps them
        for i, lw in enumerate(self.layers):
            latent = isinstance(self.shapes[i], dec.LatentLayout)
            y = self._latent_mixer(i, lw, h, rows, fb, kv, ws) if latent else self._window_mixer(i, lw, h, edges, fb, kv, ws)
            after = None if i + 1 == len(self.layers) else (one, self.layers[i + 1].norm1)
            if lw.norm2 is not None:
                h = self._step(x, dec.SublayerOut(y=y), self.hc, (one, lw.norm2), fb, lw.norm1b)
                m = ops.gate_up_silu(h, lw.wgu, self.gu_block, ops.GELU_TANH)
                h = self._step(x, dec.SublayerOut(y=ops.linear(m, lw.wd, defer_reduce=True)), self.hc, after, fb, lw.norm2b)
            else:
                h = self._step(x, dec.SublayerOut(y=y), self.hc, after, fb, lw.norm1b)
            if fb.residual_sink is not None:
                fb.residual_sink(i, x[:, 0, :c.hidden].clone())
        return ops.linear(h, self.lm_head)[:, :c.vocab_size]

    def _prefill(self, i: int, q, k, v, gate, fb: ForwardBatch, L, window: int = 0):
        if fb.kv_sink is not None:
            fb.kv_sink(i, k, v)
        pre = None if fb.prefix is None else (fb.prefix[0][i], fb.prefix[1][i], fb.prefix[2], fb.prefix[3])
        return dec.attn_gd_prefill(q, k, v, fb.seq_lens, L, self.cfg.layer_specs[i].mixer.scale, work=fb.prefill_work, prefix=pre,
                                   window=window, gate=gate)

    def _window_mixer(self, i: int, lw: ReluraxLayer, h, edges, fb: ForwardBatch, kv: PagedKVCache, ws):
        a, L, cache = self.cfg.layer_specs[i].mixer, self.shapes[i], kv.layer(i)
        q, k, v, gate = dec.conv_heads(ops.linear(h, lw.win, defer_reduce=True), fb.positions, L, self.dtype, lw.conv, lw.qnorm,
                                       lw.knorm, cache, kv.state[i], fb.slots, edges)
        if fb.is_prefill:
            o = self._prefill(i, q, k, v, gate, fb, L, a.window)
        else:
            # the step's split count is chosen for whole contexts; a window needs no more than its own
            splits = min(fb.num_splits, ops.decode_splits(a.window or self.cfg.max_position, h.shape[0], L.kv_heads, self.split_tokens))
            o = dec.attn_gd_decode(q, cache, fb.block_tables, fb.context_lens, L, a.scale, splits, ws, a.window, gate)
        return ops.linear(o, lw.wo, defer_reduce=True)

    def _latent_mixer(self, i: int, lw: ReluraxLayer, h, rows: dict, fb: ForwardBatch, kv: PagedKVCache, ws):
        a, L = self.cfg.layer_specs[i].mixer, self.shapes[i]
        src = i if L.own else a.kv_from
        cache = kv.layer(src)[0]
        cq, gate, row = dec.latent_rows(ops.linear(h, lw.win, defer_reduce=True), fb.positions, self.rot[i], L, self.dtype, lw.qnorm,
                                        lw.knorm, cache if L.own else None, fb.slots)
        q = dec.rotate_heads(ops.linear(cq, lw.wuq, defer_reduce=True), fb.positions, self.rot[i], L, self.dtype)
        if fb.is_prefill:
            if L.own:
                rows[i] = row
            T, (dk, dv) = cq.shape[0], L.pads
            k = ops.linear(rows[src], lw.wk).view(T, L.heads, dk)
            v = ops.linear(rows[src], lw.wv).view(T, L.heads, dv)
            o = self._prefill(i, q, k, v, gate, fb, L)
        else:
            o = dec.attn_latent_decode(dec.to_latent(q, lw.wabs, L), cache, fb.block_tables, fb.context_lens, L, a.scale,
                                       fb.num_splits, ws, gate)
            o = dec.from_latent(o, lw.wuv, L)
        return ops.linear(o, lw.wo, defer_reduce=True)
