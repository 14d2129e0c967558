"""Sufolix decoder on the gfx950 kernels.

The residual is S parallel fp32 streams (hyper-connections). Per layer, with the stream step
fused around every sublayer (ops/decoder.py):

    h    = norm(sum_s in_s x_s)                 HIP  (finishes the previous sublayer too)
    qkv  = h Wqkv^T                             GEMM (split-K slabs at decode)
    q,k,v = heads(qkv)                          HIP  (bias, rotation, q/k norm, value mixing, KV write)
    o    = attn(q, K, V)                        HIP  (MFMA flash prefill | split-KV paged decode)
    y    = o Wo^T                               GEMM
    x_t  = sum_s mix[s, t] x_s + out_t y        HIP  (+ the next sublayer's h)
    feed-forward: SwiGLU (GEMM + fused epilogue), or router top-k, expert GEMMs on the tokens
    scaled by their weight, and a gated shared expert
logits = norm(sum_t x_t) Wlm^T.

Weights are stored padded with zeros: the width, feature counts and head sizes to what the
tile kernels need (``ops.decoder.pad_to`` / ``head_pads``), which leaves every product
unchanged; norms divide by the true sizes. bf16 or fp32 (true 32-bit products) throughout;
residual streams, norms, router, rotation and softmax are fp32 in both.
"""
from __future__ import annotations

import math
from dataclasses import dataclass

import torch

from operator_amd import ops
from operator_amd.ops import decoder as dec
from operator_amd.parallel.comm import Group

from .base import ForwardBatch
from .config import SufolixConfig
from .kv_cache import PagedKVCache
from .padded import PaddedModel


@dataclass
class SufolixLayer:
    """One layer's tensors (fp32 where small constants, the compute dtype for the products)."""
    wqkv: torch.Tensor            # [ncol, ld] packed q | k | v rows, heads padded
    bqkv: torch.Tensor            # [ncol] fp32
    wo: torch.Tensor              # [ld, ocol]
    norm1: torch.Tensor           # [ld] fp32
    in1: torch.Tensor             # stream coefficients of the mixer, fp32: [S], [S, S], [S]
    mix1: torch.Tensor
    out1: torch.Tensor
    lam: torch.Tensor | None = None     # [1] fp32 value-mixing weight
    norm2: torch.Tensor | None = None   # feed-forward (None: the layer has none)
    in2: torch.Tensor | None = None
    mix2: torch.Tensor | None = None
    out2: torch.Tensor | None = None
    wgu: torch.Tensor | None = None     # dense [2 ff, ld] or experts [E, 2 ff, ld], 64-row interleaved
    wd: torch.Tensor | None = None      # [ld, ff] or [E, ld, ff]
    wr: torch.Tensor | None = None      # router rows, then the shared expert's gate row
    sgu: torch.Tensor | None = None     # shared expert
    sd: torch.Tensor | None = None


class SufolixModel(PaddedModel):
    LAYER = SufolixLayer
    LAYOUT_FUNCS = PaddedModel.LAYOUT_FUNCS + ("init_random", "_layer")

    def __init__(self, cfg: SufolixConfig, device: str | torch.device = "cuda", tp: Group | None = None,
                 dtype: torch.dtype = torch.bfloat16, weight_dtype: str = "bfloat16"):
        super().__init__(cfg, device, tp, dtype, weight_dtype)
        self.heads = [dec.HeadLayout(a.heads, a.kv_heads, a.dim, a.vdim, a.rot_dims, True, cfg.rms_eps)
                      for a in (sp.mixer for sp in cfg.layer_specs)]
        self.hq = max(L.heads for L in self.heads)
        self.hkv = max(L.kv_heads for L in self.heads)
        tabs: dict = {}
        self.rot = []
        for sp in cfg.layer_specs:
            key = (sp.mixer.rot_base, sp.mixer.rot_dims)
            if key not in tabs:
                tabs[key] = dec.rotary_tables(cfg.max_position, *key, device=self.device) if key[1] else None
            self.rot.append(tabs[key])
        mixing = [i for i, sp in enumerate(cfg.layer_specs) if sp.mixer.v_mix]
        self.first_mix = mixing[0] if mixing else -1

    # ------------------------------------------------------------------ engine surface
    def kv_shapes(self) -> list[tuple[int, int, int]]:
        return [(L.kv_heads, *L.pads) for L in self.heads]

    # ------------------------------------------------------------------ weights
    def _layer(self, i: int, get, has) -> SufolixLayer:
        c, sp, L, W = self.cfg, self.cfg.layer_specs[i], self.heads[i], self.cfg.hidden
        a, p = sp.mixer, f"l{i}."
        (dk, dv), H, G, S = L.pads, L.heads, L.kv_heads, c.streams

        def f32(name, shape, fill=None):
            if fill is not None and not has(name):
                return fill.to(self.device)
            return get(name, shape).float().reshape(shape).contiguous()

        def norm(name):
            return self._padded(f32(name, (W,)), self.ld)

        def hc(q):   # a single stream without stored coefficients is the plain residual
            one = torch.ones(S) if S == 1 else None
            return (f32(p + f"hc{q}.in", (S,), one), f32(p + f"hc{q}.mix", (S, S), one.view(1, 1) if S == 1 else None),
                    f32(p + f"hc{q}.out", (S,), one))

        rows, bias, at = [], torch.zeros(L.ncol, device=self.device), 0
        for n, heads, d, dp in (("q", H, a.dim, dk), ("k", G, a.dim, dk), ("v", G, a.vdim, dv)):
            w, b = get(p + "mix." + n, (heads * d, W)), f32(p + f"mix.{n}.b", (heads * d,))
            for h in range(heads):
                rows.append((at, 0, w[h * d:(h + 1) * d]))
                bias[at:at + d] = b[h * d:(h + 1) * d]
                at += dp
        wo = get(p + "mix.o", (W, H * a.vdim))
        in1, mix1, out1 = hc(1)
        lw = SufolixLayer(
            wqkv=self._put(L.ncol, self.ld, rows), bqkv=bias,
            wo=self._put(self.ld, L.ocol, [(0, h * dv, wo[:, h * a.vdim:(h + 1) * a.vdim]) for h in range(H)]),
            norm1=norm(p + "norm1"), in1=in1, mix1=mix1, out1=out1,
            lam=f32(p + "mix.vmix", (1,)) if a.v_mix and i != self.first_mix else None)
        m = sp.mlp
        if m is None:
            return lw
        lw.norm2 = norm(p + "norm2")
        lw.in2, lw.mix2, lw.out2 = hc(2)
        gu = lambda q, ff: self._gate_up(get(q + "gate", (ff, W)), get(q + "up", (ff, W)))  # noqa: E731
        if not m.experts:
            lw.wgu, lw.wd = gu(p + "mlp.", m.ff), self._down(get(p + "mlp.down", (W, m.ff)))
            return lw
        lw.wgu = torch.stack([gu(f"{p}mlp.e{e}.", m.ff) for e in range(m.experts)])
        lw.wd = torch.stack([self._down(get(f"{p}mlp.e{e}.down", (W, m.ff))) for e in range(m.experts)])
        rows = [(0, 0, get(p + "mlp.router", (m.experts, W)))]
        if m.shared_ff:
            rows.append((m.experts, 0, get(p + "mlp.shared.sg", (1, W))))
            lw.sgu = gu(p + "mlp.shared.", m.shared_ff)
            lw.sd = self._down(get(p + "mlp.shared.down", (W, m.shared_ff)))
        lw.wr = self._put(dec.router_rows(m.experts), self.ld, rows)
        return lw

    def init_random(self, seed: int = 0) -> "SufolixModel":
        """Random weights of the exact architecture: O(1) activations, streams that mix mildly."""
        def get(name, shape):
            owner, leaf = ([""] + name.split("."))[-2:]
            t = self._randn(seed, name, shape, 1.0)
            if leaf.startswith("norm"):
                return 1.0 + 0.1 * t
            if leaf in ("in", "out"):
                return (1.0 / self.cfg.streams if leaf == "in" else 1.0) + 0.1 * t
            if owner.startswith("hc"):
                return 0.05 * t + torch.eye(shape[0], dtype=t.dtype, device=t.device)
            if leaf == "vmix":
                return 0.5 + 0.1 * t
            if leaf == "b":
                return 0.2 * t
            return t if leaf == "embed" else t * (1.0 / math.sqrt(shape[-1]))

        return self._build(get, lambda name: True)

    # ------------------------------------------------------------------ forward
    def forward(self, fb: ForwardBatch, kv: PagedKVCache) -> torch.Tensor:
        """Run all layers; returns logits [n_out, vocab] for fb.logits_index rows."""
        c, dt = self.cfg, self.dtype
        first = self.layers[0]
        x, h = dec.stream_init(fb.input_ids, self.embed, c.embed_scale, c.streams, c.hidden, first.in1, first.norm1, c.rms_eps)
        ws = None
        if not fb.is_prefill and h.is_cuda:   # split-KV partials, shared by every layer
            ws = dec.attn_gd_workspace(h.shape[0], self.heads, fb.num_splits, h.device)
        v_first = None
        for i, lw in enumerate(self.layers):
            y, v_first = self._mixer(i, lw, h, v_first, fb, kv, ws)
            last = i + 1 == len(self.layers)
            after = None if last else (self.layers[i + 1].in1, self.layers[i + 1].norm1)
            hc = dec.Stream(lw.in1, lw.mix1, lw.out1)
            if lw.norm2 is not None:
                h = self._step(x, dec.SublayerOut(y=y), hc, (lw.in2, lw.norm2), fb)
                y = self._feed_forward(lw, c.layer_specs[i].mlp, h)
                hc = dec.Stream(lw.in2, lw.mix2, lw.out2)
            else:
                y = dec.SublayerOut(y=y)
            h = self._step(x, y, hc, after, fb)
            if fb.residual_sink is not None:
                fb.residual_sink(i, x[:, :, :c.hidden].sum(1))
        return ops.linear(h, self.lm_head)[:, :c.vocab_size]

    def _mixer(self, i: int, lw: SufolixLayer, h, v_first, fb: ForwardBatch, kv: PagedKVCache, ws):
        """(o-projection output, the first mixing layer's values)."""
        a, L = self.cfg.layer_specs[i].mixer, self.heads[i]
        cache = kv.layer(i)
        qkv = ops.linear(h, lw.wqkv, defer_reduce=True)
        mixed = v_first if lw.lam is not None else None
        q, k, v = dec.qkv_heads(qkv, fb.positions, self.rot[i], L, self.dtype, bias=lw.bqkv, cache=cache, slots=fb.slots,
                                want_k=fb.is_prefill, want_v=fb.is_prefill or i == self.first_mix, v_first=mixed, lam=lw.lam)
        if i == self.first_mix:
            v_first = v
        if fb.is_prefill:
            if fb.kv_sink is not None:
                fb.kv_sink(i, k, v)
            pre = None if fb.prefix is None else (fb.prefix[0][i], fb.prefix[1][i], fb.prefix[2], fb.prefix[3])
            o = dec.attn_gd_prefill(q, k, v, fb.seq_lens, L, a.scale, work=fb.prefill_work, prefix=pre)
        else:
            o = dec.attn_gd_decode(q, cache, fb.block_tables, fb.context_lens, L, a.scale, fb.num_splits, ws)
        return ops.linear(o, lw.wo, defer_reduce=True), v_first

    def _feed_forward(self, lw: SufolixLayer, m, h) -> dec.SublayerOut:
        if not m.experts:
            return dec.SublayerOut(y=ops.linear(ops.gate_up_silu(h, lw.wgu, self.gu_block), lw.wd, defer_reduce=True))
        ids, wt, gate = dec.route(h, lw.wr, m.experts, m.top, bool(m.shared_ff))
        e, epos = dec.experts(h, ids, wt, lw.wgu, lw.wd)
        y = None
        if m.shared_ff:
            y = ops.linear(ops.gate_up_silu(h, lw.sgu, self.gu_block), lw.sd, defer_reduce=True)
        return dec.SublayerOut(y=y, gate=gate, e=e, epos=epos, top=m.top)
