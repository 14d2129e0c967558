"""Ops of decoders beyond the Llama block: hyper-connection residual streams, QKV heads of any
size with rotary positions and per-head norm, heads behind short convolutions, attention over
them (full or sliding window, with per-head output gates), latent attention, routed experts, and
the fp32 forms of all of them.

As in :mod:`operator_amd.ops`: GPU tensors go to the gfx950 kernels (csrc/kernels/streams.hip,
qkv_heads.hip, conv_heads.hip, latent.hip, attn_gd_*.hip, attn_latent_decode.hip, moe.hip, f32.hip), CPU tensors to the fp32 references. Widths,
head sizes and feature counts are stored padded (``pad_to``) with zero weights, so every GEMM
meets the tile kernels' alignment whatever the model's sizes.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import reference
from ._native import kernels

# general attention work items: 128 query rows whatever the head layout (attn_gd_prefill.hip)
GD_VARIANT = 5
GD_BLOCK_Q = 128
# expert GEMMs (expert_plan): most rows per expert, on average, of each form
MOE_LIST_ROWS, MOE_64_ROWS, MOE_128_ROWS = 7, 44, 220
MOE_LIST_MAX_SLOTS = 4096   # moe.hip kMaxSlots


def pad_to(n: int, m: int) -> int:
    return -(-n // m) * m


def head_pads(dim: int, vdim: int) -> tuple[int, int]:
    """Stored sizes of a query/key head and a value head (the cache tiles' granularity)."""
    return pad_to(dim, 16), pad_to(vdim, 32)


# ---------------------------------------------------------------- hyper-connection streams
@dataclass
class Stream:
    """Coefficients of one sublayer of a hyper-connected model (fp32): how it reads the S
    residual streams (``inp`` [S]), how they mix ([S, S], [from, to]) and take its output (``out`` [S])."""
    inp: torch.Tensor
    mix: torch.Tensor
    out: torch.Tensor


@dataclass
class SublayerOut:
    """A sublayer's output as its producers left it, summed by the next stream step:
    sigmoid(gate) * y + sum_k e[row of (token, k)]; every part may be absent."""
    y: object = None                     # [T, ld] rows, or SplitK slabs
    gate: torch.Tensor | None = None     # [T] fp32 logits
    e: torch.Tensor | None = None        # [rows, ld]
    epos: torch.Tensor | None = None     # [T, top] int32 row of e; None: row t * top + k
    top: int = 0


def stream_init(ids: torch.Tensor, table: torch.Tensor, scale: float, streams: int, width: int, inp: torch.Tensor,
                w: torch.Tensor, eps: float):
    """Embedding -> (streams [T, S, ld] fp32, all equal to scale * row; the first sublayer's
    normalised input [T, ld] in the table's dtype)."""
    T, ld = ids.numel(), table.shape[1]
    x = torch.empty(T, streams, ld, dtype=torch.float32, device=ids.device)
    h = torch.empty(T, ld, dtype=table.dtype, device=ids.device)
    if ids.is_cuda:
        kernels().stream_step(x, h, width, w, eps, in_=inp, ids=ids, table=table, emb_scale=scale)
    else:
        x.copy_((reference.embedding(ids, table).float() * scale)[:, None])
        h.copy_(reference.stream_norm(x, inp, w, width, eps))
    return x, h


def stream_step(x: torch.Tensor, o: SublayerOut, hc: Stream, nxt: torch.Tensor | None, w: torch.Tensor, width: int,
                eps: float, dtype: torch.dtype, rows: torch.Tensor | None = None, write_x: bool = True,
                post_w: torch.Tensor | None = None) -> torch.Tensor:
    """Finish a sublayer (``hc`` with its output ``o``) and return the next one's normalised
    input: ``nxt`` are its stream coefficients, None the plain sum at the model's end, where
    ``rows`` picks the rows wanted and ``write_x`` False leaves the streams alone. ``post_w``: weight
    of an RMS norm of the output itself before it joins (one stream)."""
    from . import SplitK

    n = x.shape[0] if rows is None else rows.numel()
    if not x.is_cuda:
        y = reference.sublayer_out(o.y, o.gate, o.e, o.epos, o.top, x.shape[0], x.shape[2])
        if post_w is not None:
            y = reference.rms_rows(y, post_w, width, eps)
        xn = reference.stream_mix(x, y, hc.mix, hc.out)
        if write_x:
            x.copy_(xn)
        if rows is not None:
            xn = xn[rows]
        return reference.stream_norm(xn, nxt, w, width, eps).to(dtype)
    h = torch.empty(n, x.shape[2], dtype=dtype, device=x.device)
    slab = isinstance(o.y, SplitK)
    kernels().stream_step(x, h, width, w, eps, in_=nxt, y=None if slab else o.y, slabs=o.y.p if slab else None,
                          splits=o.y.S if slab else 1, gate=o.gate, e=o.e, epos=o.epos, top=o.top, mix=hc.mix,
                          out=hc.out, rows=rows, write_x=write_x, post_w=post_w)
    return h


# ---------------------------------------------------------------- attention, any head size
@dataclass(frozen=True)
class HeadLayout:
    """Shapes and constants of one attention layer (true sizes; the rows hold padded ones)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    rot_dims: int = 0
    norm: bool = True      # q, k divided by their root mean square after rotation
    eps: float = 1e-6

    @property
    def pads(self) -> tuple[int, int]:
        return head_pads(self.dim, self.vdim)

    @property
    def ncol(self) -> int:
        """Columns of the packed QKV projection."""
        dk, dv = self.pads
        return pad_to((self.heads + self.kv_heads) * dk + self.kv_heads * dv, 64)

    @property
    def ocol(self) -> int:
        """Columns of the attention output the o-projection reads."""
        return pad_to(self.heads * self.pads[1], 64)


def rotary_tables(max_pos: int, base: float, dims: int, device=None) -> tuple[torch.Tensor, torch.Tensor]:
    """cos / sin [max_pos, dims / 2 padded to 4] of position * base^(-2 i / dims), fp32 from fp64 angles."""
    n = dims // 2
    inv = 1.0 / (base ** (torch.arange(n, dtype=torch.float64) * 2.0 / dims))
    a = torch.zeros(max_pos, pad_to(max(n, 1), 4), dtype=torch.float64)
    a[:, :n] = torch.outer(torch.arange(max_pos, dtype=torch.float64), inv)
    return a.cos().float().to(device), a.sin().float().to(device)


def qkv_heads(qkv, pos: torch.Tensor, rot: tuple | None, L: HeadLayout, dtype: torch.dtype, bias: torch.Tensor | None = None,
              cache: tuple | None = None, slots: torch.Tensor | None = None, want_k: bool = True, want_v: bool = True,
              v_first: torch.Tensor | None = None, lam: torch.Tensor | None = None):
    """Packed projection rows (or SplitK slabs) -> (q [T, H, dk], k [T, G, dk] | None,
    v [T, G, dv] | None) rotated, normalised and mixed with ``v_first``, k / v also written to
    the paged ``cache`` at ``slots`` (< 0: not cached)."""
    from . import SplitK

    T, dev = pos.numel(), pos.device
    dk, dv = L.pads
    cos, sin = rot if rot is not None else (None, None)
    if not pos.is_cuda:
        q, k, v = reference.qkv_heads(qkv, bias, pos, cos, sin, L, v_first, lam)
        q, k, v = q.to(dtype), k.to(dtype), v.to(dtype)
        if cache is not None:
            reference.cache_rows(cache[0], cache[1], k, v, slots)
        return q, k if want_k else None, v if want_v else None
    q = torch.empty(T, L.heads, dk, dtype=dtype, device=dev)
    k = torch.empty(T, L.kv_heads, dk, dtype=dtype, device=dev) if want_k else None
    v = torch.empty(T, L.kv_heads, dv, dtype=dtype, device=dev) if want_v else None
    slab = isinstance(qkv, SplitK)
    kc, vc = cache if cache is not None else (None, None)
    kernels().qkv_heads(q if slab else qkv, qkv.p if slab else None, qkv.S if slab else 1, bias, pos, cos, sin,
                        L.rot_dims // 2 if rot is not None else 0, L.heads, L.kv_heads, L.dim, L.norm, L.eps, v_first,
                        lam, q, k, v, kc, vc, slots, dv, L.ncol)
    return q, k, v


def _o_rows(T: int, L: HeadLayout, dtype, dev) -> torch.Tensor:
    o = torch.empty(T, L.ocol, dtype=dtype, device=dev)
    used = L.heads * L.pads[1]
    if used < L.ocol:
        o[:, used:].zero_()
    return o


def attn_gd_prefill(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, seq_lens: list[int], L: HeadLayout, scale: float,
                    work: tuple | None = None, prefix: tuple | None = None, window: int = 0,
                    gate: torch.Tensor | None = None) -> torch.Tensor:
    """Causal attention over packed sequences -> [T, ocol] rows for the o-projection. ``window``: a
    query sees keys less than that far back (0: all); ``gate`` [T, H] fp32 scales every head's output.
    ``work`` = (cu_seqlens, work_seq, work_q0, GD_VARIANT); ``prefix`` as in ``attn_prefill``."""
    if not q.is_cuda:
        cu = [0]
        for n in seq_lens:
            cu.append(cu[-1] + int(n))
        r = reference.attn_prefill(q, k, v, cu, scale, prefix=None if prefix is None else (prefix[0], prefix[1], prefix[3]),
                                   window=window)
        r = r if gate is None else (r.float() * gate[..., None]).to(r.dtype)
        o = torch.zeros(q.shape[0], L.ocol, dtype=q.dtype)
        o[:, :L.heads * L.pads[1]] = r.reshape(q.shape[0], -1)
        return o
    if work is None:
        from . import prefill_work_list

        cu = [0]
        for n in seq_lens:
            cu.append(cu[-1] + int(n))
        ws, wq = prefill_work_list([int(n) for n in seq_lens], GD_BLOCK_Q)
        work = tuple(torch.tensor(t, dtype=torch.int32, device=q.device) for t in (cu, ws, wq)) + (GD_VARIANT,)
    if work[3] != GD_VARIANT:
        raise ValueError("attn_gd_prefill needs a work list cut at GD_BLOCK_Q rows")
    o = _o_rows(q.shape[0], L, q.dtype, q.device)
    pk, pv, sp = (None, None, None) if prefix is None else prefix[:3]
    kernels().attn_gd_prefill(q, k, v, o, work[0], work[1], work[2], scale, pk, pv, sp, window, gate)
    return o


def attn_gd_workspace(B: int, layouts, num_splits: int, device):
    """fp32 partials of split decode attention, shared by a model's layers (None: one split)."""
    if num_splits <= 1:
        return None
    n = max(B * L.heads * num_splits * (L.rp if isinstance(L, LatentLayout) else L.pads[1]) for L in layouts)
    m = max(B * L.heads * num_splits * 2 for L in layouts)
    return (torch.empty(n, dtype=torch.float32, device=device), torch.empty(m, dtype=torch.float32, device=device))


def attn_gd_decode(q: torch.Tensor, cache: tuple, block_tables: torch.Tensor, seq_lens: torch.Tensor, L: HeadLayout,
                   scale: float, num_splits: int = 1, workspace: tuple | None = None, window: int = 0,
                   gate: torch.Tensor | None = None) -> torch.Tensor:
    """One query token per sequence over the paged cache -> [B, ocol] rows (``window``, ``gate``: as in
    ``attn_gd_prefill``)."""
    if not q.is_cuda:
        r = reference.attn_decode_rows(q, cache[0], cache[1], block_tables, seq_lens, scale, window)
        r = r if gate is None else (r.float() * gate[..., None]).to(r.dtype)
        o = torch.zeros(q.shape[0], L.ocol, dtype=q.dtype)
        o[:, :L.heads * L.pads[1]] = r.reshape(q.shape[0], -1)
        return o
    o = _o_rows(q.shape[0], L, q.dtype, q.device)
    if num_splits > 1 and workspace is None:
        workspace = attn_gd_workspace(q.shape[0], [L], num_splits, q.device)
    ws = workspace if num_splits > 1 else (None, None)
    kernels().attn_gd_decode(q, cache[0], cache[1], block_tables, seq_lens, o, ws[0], ws[1], num_splits, scale, window, gate)
    return o


# ---------------------------------------------------------------- heads behind short convolutions
@dataclass
class SequenceEdges:
    """Where a step's rows stand in their sequences. A prefill has ``cu`` (device, the GPU) /
    ``lens`` (host, the CPU) of its packed sequences and ``prev_pages`` [S] int32, the page of the
    tokens before a sequence's first row (-1 or None: there are none); a decode step ``block_tables``."""
    cu: torch.Tensor | None = None
    lens: list | None = None
    prev_pages: torch.Tensor | None = None
    block_tables: torch.Tensor | None = None


def conv_ncol(L: HeadLayout) -> int:
    """Columns of a packed query | key | gate projection."""
    return pad_to((L.heads + L.kv_heads) * L.pads[0] + L.heads, 64)


def conv_heads(x, pos: torch.Tensor, L: HeadLayout, dtype: torch.dtype, conv: torch.Tensor, qw: torch.Tensor, kw: torch.Tensor,
               cache: tuple, tails: torch.Tensor | None, slots: torch.Tensor, edges: SequenceEdges):
    """Packed q | k | gate rows (or SplitK slabs) -> (q [T, H, dk], k [T, G, dk], v [T, G, dv], gate [T, H]
    fp32): q and k through the short causal convolution ``conv`` [taps, (H + G) dk] and a weighted
    per-head RMS norm (weights in ``dtype``), v the convolved key without the norm, gate the sigmoid. k / v (None at decode)
    also go to the paged ``cache``, and the last taps - 1 projected rows to ``tails`` [pages, taps - 1, C]."""
    from . import SplitK

    T, dev = pos.numel(), pos.device
    dk, dv = L.pads
    if not pos.is_cuda:
        q, k, v, gate = reference.conv_heads(x, pos, L, conv, qw, kw, tails, slots, edges, cache[0].shape[2])
        q, k, v = q.to(dtype), k.to(dtype), v.to(dtype)
        reference.cache_rows(cache[0], cache[1], k, v, slots)
        return q, k, v, gate
    prefill = edges.block_tables is None
    q = torch.empty(T, L.heads, dk, dtype=dtype, device=dev)
    k = torch.empty(T, L.kv_heads, dk, dtype=dtype, device=dev) if prefill else None
    v = torch.empty(T, L.kv_heads, dv, dtype=dtype, device=dev) if prefill else None
    gate = torch.empty(T, L.heads, dtype=torch.float32, device=dev)
    slab = isinstance(x, SplitK)
    kernels().conv_heads(q if slab else x, x.p if slab else None, x.S if slab else 1, conv, qw, kw, pos, L.dim, L.eps, q, k, v,
                         cache[0], cache[1], slots, tails, gate, conv_ncol(L), edges.cu if prefill else None,
                         edges.prev_pages if prefill else None, edges.block_tables)
    return q, k, v, gate


# ---------------------------------------------------------------- latent attention
@dataclass(frozen=True)
class LatentLayout:
    """Shapes of one latent-attention layer (true sizes): ``heads`` of ``dim`` unrotated and ``rot``
    rotated query / key dimensions and ``vdim`` value ones, queries from a latent of ``q_rank``, keys
    and values from one of ``kv_rank``; ``own`` False: it reads another layer's latent rows."""
    heads: int
    dim: int
    rot: int
    vdim: int
    q_rank: int
    kv_rank: int
    own: bool = True
    eps: float = 1e-6

    @property
    def pads(self) -> tuple[int, int]:
        """Stored sizes of an expanded query / key head and a value head."""
        return head_pads(self.dim + self.rot, self.vdim)

    @property
    def qp(self) -> int:
        return max(128, pad_to(self.q_rank, 64))

    @property
    def rp(self) -> int:
        return pad_to(self.kv_rank, 32)

    @property
    def rotp(self) -> int:
        return pad_to(self.rot, 8)

    @property
    def ck(self) -> int:
        """Columns of a cached row: latent (rp), rotated part, zeros."""
        return max(128, pad_to(self.rp + self.rot, 64))

    @property
    def ncol(self) -> int:
        """Columns of the packed projection: query latent, latent, rotated part, gates."""
        return pad_to(self.qp + (self.rp + self.rotp if self.own else 0) + self.heads, 64)

    @property
    def ocol(self) -> int:
        return pad_to(self.heads * self.pads[1], 64)


def latent_rows(x, pos: torch.Tensor, rot: tuple, L: LatentLayout, dtype: torch.dtype, qw: torch.Tensor, cw: torch.Tensor | None,
                cache: torch.Tensor | None, slots: torch.Tensor):
    """Packed projection -> (normed query latent [T, qp], gate [T, H] fp32, latent rows [T, ck] | None); the
    rows also go to the paged ``cache`` [pages, 1, P, ck]."""
    from . import SplitK

    T, dev = pos.numel(), pos.device
    if not pos.is_cuda:
        return reference.latent_rows(x, pos, rot, L, dtype, qw, cw, cache, slots)
    cq = torch.empty(T, L.qp, dtype=dtype, device=dev)
    gate = torch.empty(T, L.heads, dtype=torch.float32, device=dev)
    lat = torch.empty(T, L.ck, dtype=dtype, device=dev) if L.own else None
    slab = isinstance(x, SplitK)
    kernels().latent_rows(cq if slab else x, x.p if slab else None, x.S if slab else 1, L.ncol, L.q_rank, L.kv_rank, L.rp, L.rot,
                          L.rotp, qw, cw, L.eps, pos, rot[0], rot[1], cq, lat, cache if L.own else None, slots if L.own else None, gate)
    return cq, gate, lat


def rotate_heads(q, pos: torch.Tensor, rot: tuple, L: LatentLayout, dtype: torch.dtype) -> torch.Tensor:
    """Query heads [T, H dk] (rows, rotated in place, or SplitK slabs) -> [T, H, dk] with the columns dim ..
    dim + rot of every head rotated (first half paired with the second)."""
    from . import SplitK

    T, dk = pos.numel(), L.pads[0]
    if not pos.is_cuda:
        return reference.rotate_heads(q.view(T, L.heads, dk), pos, rot, L.dim, L.rot).to(dtype)
    slab = isinstance(q, SplitK)
    out = torch.empty(T, L.heads, dk, dtype=dtype, device=pos.device) if slab else q.view(T, L.heads, dk)
    kernels().rotate_heads(out, q.p if slab else None, q.S if slab else 1, L.dim, L.rot, pos, rot[0], rot[1])
    return out


def to_latent(q: torch.Tensor, w: torch.Tensor, L: LatentLayout) -> torch.Tensor:
    """Decode queries in the space of the cached rows: [B, H, dk] -> [B, H, ck], ``w`` [H, rp, pad16(dim)] the
    transposed key expansion of every head."""
    if not q.is_cuda:
        y = torch.zeros(q.shape[0], L.heads, L.ck, dtype=q.dtype)
        y[..., :L.rp] = reference.head_gemm(q[..., :w.shape[2]], w)
        y[..., L.rp:L.rp + L.rot] = q[..., L.dim:L.dim + L.rot]
        return y
    if q.dtype == torch.float32:
        y = torch.zeros(q.shape[0], L.heads, L.ck, dtype=q.dtype, device=q.device)
        kernels().head_gemm(q, w, y)
        y[..., L.rp:L.rp + L.rot] = q[..., L.dim:L.dim + L.rot]
        return y
    y = torch.empty(q.shape[0], L.heads, L.ck, dtype=q.dtype, device=q.device)
    kernels().head_gemm(q, w, y, L.dim, L.rot)
    return y


def from_latent(o: torch.Tensor, w: torch.Tensor, L: LatentLayout) -> torch.Tensor:
    """Attention outputs in the latent space [B, H, rp] -> [B, ocol] rows of values (``w`` [H, dv, rp])."""
    y = _o_rows(o.shape[0], L, o.dtype, o.device)
    if not o.is_cuda:
        y[:, :L.heads * L.pads[1]] = reference.head_gemm(o, w).reshape(o.shape[0], -1)
        return y
    kernels().head_gemm(o, w, y)
    return y


def attn_latent_decode(q: torch.Tensor, cache: torch.Tensor, block_tables: torch.Tensor, seq_lens: torch.Tensor, L: LatentLayout,
                       scale: float, num_splits: int = 1, workspace: tuple | None = None,
                       gate: torch.Tensor | None = None) -> torch.Tensor:
    """One query token per sequence over cached latent rows: [B, H, rp] sums of the latents, gated."""
    if not q.is_cuda:
        r = reference.attn_decode_rows(q, cache, cache[..., :L.rp], block_tables, seq_lens, scale)
        return r if gate is None else (r.float() * gate[..., None]).to(r.dtype)
    o = torch.empty(q.shape[0], L.heads, L.rp, dtype=q.dtype, device=q.device)
    if num_splits > 1 and workspace is None:
        n = q.shape[0] * L.heads * num_splits
        workspace = (torch.empty(n * L.rp, dtype=torch.float32, device=q.device),
                     torch.empty(2 * n, dtype=torch.float32, device=q.device))
    ws = workspace if num_splits > 1 else (None, None)
    kernels().attn_latent_decode(q, cache, block_tables, seq_lens, o.view(q.shape[0], -1), L.rp, ws[0], ws[1], num_splits, scale, gate)
    return o


# ---------------------------------------------------------------- routed experts
def router_rows(experts: int) -> int:
    """Stored rows of a router with a gate row: whole groups of 1, 2 or 4 MFMA tiles."""
    n = pad_to(experts + 1, 16)
    return n if n <= 32 else pad_to(n, 64)


def route(h: torch.Tensor, wr: torch.Tensor, experts: int, top: int, gated: bool):
    """Router: (ids [T, top] int32, weights [T, top] fp32 sigmoid scores of the largest logits,
    gate [T] fp32 | None). ``wr`` rows: the experts', then (``gated``) the shared expert's gate,
    then zeros (``router_rows``); logits in fp32."""
    T, dev = h.shape[0], h.device
    if not h.is_cuda:
        return reference.route(h, wr, experts, top, gated)
    ids = torch.empty(T, top, dtype=torch.int32, device=dev)
    wt = torch.empty(T, top, dtype=torch.float32, device=dev)
    gate = torch.empty(T, dtype=torch.float32, device=dev) if gated else None
    if h.dtype == torch.bfloat16:
        kernels().moe_route(h, wr, experts, ids, wt, gate)
    else:
        z = torch.empty(T, wr.shape[0], dtype=torch.float32, device=dev)
        kernels().gemm_f32(h, wr, z)
        kernels().moe_topk(z, experts, ids, wt, gate)
    return ids, wt, gate


def expert_rows_bound(slots: int, experts: int, bm: int) -> int:
    """Rows an expert-sorted batch can need: every segment padded to ``bm``."""
    return pad_to(slots + min(experts, slots) * (bm - 1), bm)


def expert_plan(slots: int, E: int) -> int:
    """How bf16 expert GEMMs run, by the rows an expert gets on average: 0 = weights streamed
    against the rows of each expert's own list, no sorting (few rows), 64 / 128 = sorted rows in
    tiles of that many on the decode GEMM, 256 = the prefill tile kernel."""
    rows = slots / E
    if rows <= MOE_LIST_ROWS and slots <= MOE_LIST_MAX_SLOTS:
        return 0
    return 64 if rows <= MOE_64_ROWS else 128 if rows <= MOE_128_ROWS else 256


def experts(h: torch.Tensor, ids: torch.Tensor, wt: torch.Tensor, wgu: torch.Tensor, wd: torch.Tensor,
            plan: int | None = None):
    """SwiGLU experts on their tokens scaled by the router weight: (rows, epos) such that
    token t's contributions are rows[epos[t, k]] (epos None: row t * top + k).
    wgu [E, 2 ff, ld] with gate | up interleaved in 64-row blocks, wd [E, ld, ff];
    ``plan``: expert_plan's choice (bf16), for tests and tuning."""
    T, top = ids.shape
    E, ld, ff = wd.shape
    slots = T * top
    if not h.is_cuda:
        return reference.experts(h, ids, wt, wgu, wd), None
    C, dev = kernels(), h.device
    bf16 = h.dtype == torch.bfloat16
    bm = (expert_plan(slots, E) if plan is None else plan) if bf16 else 64
    if bm in (64, 128) and bf16 and ld % 128:
        bm = 256   # the decode GEMM's column tiles
    if bm == 0:
        m = torch.empty(slots, ff, dtype=h.dtype, device=dev)
        C.moe_gemm_skinny(h, wgu, m, ids, wt, top, True)
        y = torch.empty(slots, ld, dtype=h.dtype, device=dev)
        C.moe_gemm_skinny(m, wd, y, ids, wt, 1, False)
        return y, None
    rows = expert_rows_bound(slots, E, bm)
    i32 = dict(dtype=torch.int32, device=dev)
    pos, src, gtab = torch.empty(T, top, **i32), torch.empty(rows, **i32), torch.empty(1 + rows // bm, **i32)
    rs = torch.empty(rows, dtype=torch.float32, device=dev)
    C.moe_sort(ids, wt, E, bm, pos, src, rs, gtab)
    m = torch.empty(rows, ff, dtype=h.dtype, device=dev)
    y = torch.empty(rows, ld, dtype=h.dtype, device=dev)
    if bf16 and bm < 256:
        C.moe_gemm_rows(h, wgu, m, bm, gtab, src, rs, True)
        C.moe_gemm_rows(m, wd, y, bm, gtab)
        return y, pos
    xp = torch.empty(rows, ld, dtype=h.dtype, device=dev)
    C.moe_gather(h, src, gtab, bm, xp)
    if bf16:
        C.moe_gemm_tile(xp, wgu, m, gtab, rs, True)
        C.moe_gemm_tile(m, wd, y, gtab)
    else:
        C.gemm_f32(xp, wgu, m, True, gtab, rs)
        C.gemm_f32(m, wd, y, False, gtab)
    return y, pos
