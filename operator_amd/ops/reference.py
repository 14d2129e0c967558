"""Plain-PyTorch fp32 reference implementations of every HIP kernel.

These define the numerics each gfx950 kernel is tested against (tests/test_kernels_gpu.py)
and are what runs when a model is executed on CPU (the CPU test tier, gloo
multi-process TP tests). They are intentionally simple and unfused.
"""
from __future__ import annotations

import math

import torch


def rmsnorm(x: torch.Tensor, w: torch.Tensor, eps: float, residual: torch.Tensor | None = None):
    """y = rmsnorm(x [+ residual]); returns (y, new_residual). HF Llama numerics."""
    if residual is not None:
        x = (x.float() + residual.float()).to(x.dtype)
        new_res = x
    else:
        new_res = None
    xf = x.float()
    var = xf.pow(2).mean(-1, keepdim=True)
    y = (xf * torch.rsqrt(var + eps)).to(x.dtype)
    return (y.float() * w.float()).to(x.dtype), new_res


def silu_mul(gu: torch.Tensor, block: int | None = None, gelu: bool = False) -> torch.Tensor:
    """silu(gate) * up (``gelu``: tanh-gelu instead); gate|up columns interleaved in blocks of ``block`` features
    (None: the plain [gate | up] concatenation)."""
    inter = gu.shape[-1] // 2
    if block and block != inter:
        v = gu.reshape(*gu.shape[:-1], inter // block, 2, block)
        g, u = v[..., 0, :].reshape(*gu.shape[:-1], inter), v[..., 1, :].reshape(*gu.shape[:-1], inter)
    else:
        g, u = gu[..., :inter], gu[..., inter:]
    F = torch.nn.functional
    s = (F.gelu(g.float(), approximate="tanh") if gelu else F.silu(g.float())).to(gu.dtype)
    return (s.float() * u.float()).to(gu.dtype)


def embedding(ids: torch.Tensor, table: torch.Tensor) -> torch.Tensor:
    return table[ids.clamp(0, table.shape[0] - 1)]


def rope_tables(max_pos: int, head_dim: int, theta: float, scaling: dict | None = None,
                device=None) -> tuple[torch.Tensor, torch.Tensor]:
    """fp32 cos/sin tables [max_pos, head_dim/2]; supports Llama-3.1 'llama3' scaling."""
    inv = 1.0 / (theta ** (torch.arange(0, head_dim, 2, dtype=torch.float64) / head_dim))
    if scaling and scaling.get("rope_type", scaling.get("type")) == "llama3":
        factor = scaling["factor"]
        lo, hi = scaling.get("low_freq_factor", 1.0), scaling.get("high_freq_factor", 4.0)
        old = scaling.get("original_max_position_embeddings", 8192)
        lo_wl, hi_wl = old / lo, old / hi
        wl = 2 * math.pi / inv
        smooth = (old / wl - lo) / (hi - lo)
        scaled = torch.where(wl > lo_wl, inv / factor, inv)
        mid = (wl <= lo_wl) & (wl >= hi_wl)
        inv = torch.where(mid, (1 - smooth) * inv / factor + smooth * inv, scaled)
    t = torch.arange(max_pos, dtype=torch.float64)
    f = torch.outer(t, inv)
    return f.cos().float().to(device), f.sin().float().to(device)


def apply_rope(x: torch.Tensor, pos: torch.Tensor, cos: torch.Tensor, sin: torch.Tensor) -> torch.Tensor:
    """x: [T, H, D] -> rotate-half RoPE at positions pos [T]."""
    half = x.shape[-1] // 2
    c = cos[pos].unsqueeze(1)
    s = sin[pos].unsqueeze(1)
    xf = x.float()
    x1, x2 = xf[..., :half], xf[..., half:]
    return torch.cat([x1 * c - x2 * s, x2 * c + x1 * s], dim=-1).to(x.dtype)


K_TILE = 16  # tokens per K-cache tile


def k_tile_index(D: int = 128) -> torch.Tensor:
    """Physical offset inside a [16 tokens x D] K-cache tile of logical element (t, d).

    K is stored so that each MFMA fragment load of the decode-attention kernel is
    one contiguous 1 KB wave access: a tile is [ks 4][lg 4][token 16][8 dims]
    with d = 32*lg + 8*ks + j (lg = lane >> 4 group, ks = k-step) — instead of
    16 token rows x 64 B per instruction. V keeps the row layout."""
    t = torch.arange(K_TILE)[:, None]
    d = torch.arange(D)[None, :]
    lg, ks, j = d // 32, (d % 32) // 8, d % 8
    return ((ks * 4 + lg) * K_TILE + t) * 8 + j


def k_cache_logical(k_cache: torch.Tensor) -> torch.Tensor:
    """[pages, Hkv, P, D] tiled K cache -> logical (token-row) copy."""
    pages, Hkv, P, D = k_cache.shape
    idx = k_tile_index(D).flatten().to(k_cache.device)
    return k_cache.reshape(pages, Hkv, P // K_TILE, K_TILE * D)[..., idx].reshape(pages, Hkv, P, D)


def k_cache_write(k_cache: torch.Tensor, page: int, off: int, k: torch.Tensor) -> None:
    """k_cache[page, :, off] = k ([Hkv, D]) in the tiled K layout."""
    pages, Hkv, P, D = k_cache.shape
    idx = k_tile_index(D)[off % K_TILE].to(k_cache.device)
    k_cache.view(pages, Hkv, P // K_TILE, K_TILE * D)[page, :, off // K_TILE, idx] = k


FP8_KV_MAX = 448.0  # OCP e4m3fn


def kv_store(x: torch.Tensor, cache_dtype: torch.dtype, scale: float) -> torch.Tensor:
    """Value as held by a cache of ``cache_dtype``: as is, or e4m3fn(x / scale) saturated."""
    if cache_dtype == torch.float8_e4m3fn:
        return (x.float() / scale).clamp(-FP8_KV_MAX, FP8_KV_MAX).to(torch.float8_e4m3fn)
    return x.to(cache_dtype)


def kv_load(c: torch.Tensor, scale: float) -> torch.Tensor:
    """fp32 view of cache contents (fp8 caches dequantised by their scale)."""
    return c.float() * scale if c.dtype == torch.float8_e4m3fn else c.float()


def rope_kv(qkv: torch.Tensor, pos: torch.Tensor, cos: torch.Tensor, sin: torch.Tensor, Hq: int, Hkv: int,
            k_cache: torch.Tensor | None = None, v_cache: torch.Tensor | None = None,
            slots: torch.Tensor | None = None, k_scale: float = 1.0, v_scale: float = 1.0):
    """Split packed qkv, rotate q/k, optionally scatter k/v into the paged cache.

    Cache layout [pages, Hkv, page, D] (K tiled, see k_tile_index; V row-major);
    slot = page*page_size + offset; slot < 0 skips.
    Returns (q [T,Hq,D], k [T,Hkv,D], v [T,Hkv,D]).
    """
    T = qkv.shape[0]
    D = cos.shape[1] * 2
    q = qkv[:, : Hq * D].reshape(T, Hq, D)
    k = qkv[:, Hq * D: (Hq + Hkv) * D].reshape(T, Hkv, D)
    v = qkv[:, (Hq + Hkv) * D:].reshape(T, Hkv, D)
    q = apply_rope(q, pos, cos, sin)
    k = apply_rope(k, pos, cos, sin)
    if k_cache is not None:
        P = k_cache.shape[2]
        for t in range(T):
            s = int(slots[t])
            if s < 0:
                continue
            k_cache_write(k_cache, s // P, s % P, kv_store(k[t], k_cache.dtype, k_scale))
            v_cache[s // P, :, s % P] = kv_store(v[t], v_cache.dtype, v_scale)
    return q, k.contiguous(), v.contiguous()


def attn_prefill(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, cu_seqlens: list[int] | torch.Tensor,
                 scale: float, prefix: tuple | None = None, window: int = 0) -> torch.Tensor:
    """Causal GQA attention over packed variable-length sequences. q [T,Hq,D], k/v [T,Hkv,D].
    ``prefix`` = (pk, pv, lens): sequence i's keys start with the rows pk[:lens[i]] /
    pv[:lens[i]] (a cached shared prompt prefix), visible to all of its query rows. ``window``: only
    keys less than that far back (0: all)."""
    cu = [int(x) for x in cu_seqlens]
    Hq, Hkv = q.shape[1], k.shape[1]
    G = Hq // Hkv
    out = torch.zeros(q.shape[0], Hq, v.shape[2], dtype=q.dtype, device=q.device)
    for i in range(len(cu) - 1):
        a, b = cu[i], cu[i + 1]
        if b == a:
            continue
        pl = int(prefix[2][i]) if prefix is not None else 0
        kk, vv = k[a:b], v[a:b]
        if pl:
            kk, vv = torch.cat([prefix[0][:pl].to(k.dtype), kk]), torch.cat([prefix[1][:pl].to(v.dtype), vv])
        qs = q[a:b].float().transpose(0, 1)                      # [Hq, L, D]
        ks = kk.float().transpose(0, 1).repeat_interleave(G, 0)
        vs = vv.float().transpose(0, 1).repeat_interleave(G, 0)
        s = torch.matmul(qs, ks.transpose(1, 2)) * scale
        L = b - a
        mask = torch.ones(L, L, dtype=torch.bool, device=q.device).triu(1)
        if pl:
            mask = torch.cat([torch.zeros(L, pl, dtype=torch.bool, device=q.device), mask], 1)
        if window:
            i, j = torch.arange(L, device=q.device)[:, None] + pl, torch.arange(L + pl, device=q.device)[None]
            mask |= i - j >= window
        s.masked_fill_(mask, float("-inf"))
        p = torch.softmax(s, -1)
        out[a:b] = torch.matmul(p, vs).transpose(0, 1).to(q.dtype)
    return out


def attn_decode(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, block_tables: torch.Tensor,
                seq_lens: torch.Tensor, scale: float, k_scale: float = 1.0, v_scale: float = 1.0) -> torch.Tensor:
    """One query token per sequence over a paged cache [pages, Hkv, page, D] (K tiled;
    bf16, or e4m3fn holding x / scale)."""
    B, Hq, D = q.shape
    Hkv, P = k_cache.shape[1], k_cache.shape[2]
    k_cache = k_cache_logical(k_cache)
    G = Hq // Hkv
    out = torch.zeros_like(q)
    for b in range(B):
        L = int(seq_lens[b])
        if L == 0:
            continue
        npg = (L + P - 1) // P
        pages = block_tables[b, :npg].long()
        ks = kv_load(k_cache[pages].permute(1, 0, 2, 3).reshape(Hkv, npg * P, D)[:, :L], k_scale)
        vs = kv_load(v_cache[pages].permute(1, 0, 2, 3).reshape(Hkv, npg * P, D)[:, :L], v_scale)
        ks = ks.repeat_interleave(G, 0)
        vs = vs.repeat_interleave(G, 0)
        s = torch.einsum("hd,hld->hl", q[b].float(), ks) * scale
        p = torch.softmax(s, -1)
        out[b] = torch.einsum("hl,hld->hd", p, vs).to(q.dtype)
    return out


def gumbel_noise_ref(seed: int, position: int, vocab: int, col_offset: int = 0) -> torch.Tensor:
    """Host mirror of the device counter hash (common.h mix64 / hash_col / uniform01), vectorised."""
    import numpy as np

    M = (1 << 64) - 1
    k = ((seed * 0x9E3779B97F4A7C15) & M) ^ ((position << 32) & M)
    k ^= k >> 33
    k = (k * 0xFF51AFD7ED558CCD) & M
    k ^= k >> 33
    k = (k * 0xC4CEB9FE1A85EC53) & M
    k ^= k >> 33
    k1, k2 = np.uint32(k & 0xFFFFFFFF), np.uint32(k >> 32)
    with np.errstate(over="ignore"):
        h = (np.arange(vocab, dtype=np.uint64) + np.uint64(col_offset & 0xFFFFFFFF)).astype(np.uint32) ^ k1
        h ^= h >> np.uint32(16)
        h *= np.uint32(0x7FEB352D)
        h ^= h >> np.uint32(15)
        h ^= k2
        h *= np.uint32(0x846CA68B)
        h ^= h >> np.uint32(16)
    u = (h >> np.uint32(9)).astype(np.float64) + 0.5
    u = torch.from_numpy(u / 8388608.0)
    return -torch.log(-torch.log(u))


def sample_shard(logits: torch.Tensor, temperature: torch.Tensor, seeds: torch.Tensor, positions: torch.Tensor,
                 col_offset: int = 0) -> tuple[torch.Tensor, torch.Tensor]:
    """Greedy when T<=0 else Gumbel-max with the same counter hash as the kernel.

    Returns (global token ids, winning perturbed values) for a vocab shard.
    """
    out = torch.empty(logits.shape[0], dtype=torch.long)
    val = torch.empty(logits.shape[0], dtype=torch.float32)
    for r in range(logits.shape[0]):
        x = logits[r].double().cpu()
        t = float(temperature[r])
        if t > 0:
            x = x / t + gumbel_noise_ref(int(seeds[r]), int(positions[r]), x.numel(), col_offset)
        i = int(torch.argmax(x))
        out[r] = i + col_offset
        val[r] = float(x[i])
    return out.to(logits.device), val.to(logits.device)


def sample(logits: torch.Tensor, temperature: torch.Tensor, seeds: torch.Tensor,
           positions: torch.Tensor) -> torch.Tensor:
    return sample_shard(logits, temperature, seeds, positions)[0]


# ---------------------------------------------------------------- ops/decoder.py
def stream_norm(x: torch.Tensor, inp: torch.Tensor | None, w: torch.Tensor, width: int, eps: float) -> torch.Tensor:
    """RMS norm of the weighted (``inp`` None: plain) sum of the streams [T, S, ld]; fp32."""
    u = x.sum(1) if inp is None else torch.matmul(x.transpose(1, 2), inp)
    return u * torch.rsqrt(u.pow(2).sum(-1, keepdim=True) / width + eps) * w


def stream_mix(x: torch.Tensor, y: torch.Tensor, mix: torch.Tensor, out: torch.Tensor) -> torch.Tensor:
    """New streams: x'_t = sum_s mix[s, t] x_s + out[t] y."""
    return torch.matmul(mix.t(), x) + out[None, :, None] * y[:, None, :]


def sublayer_out(y, gate, e, epos, top: int, T: int, ld: int) -> torch.Tensor:
    """A sublayer's output in fp32 from its parts (ops.decoder.SublayerOut)."""
    r = torch.zeros(T, ld) if y is None else y.float()
    if gate is not None:
        r = r * torch.sigmoid(gate)[:, None]
    if top:
        rows = torch.arange(T * top).view(T, top) if epos is None else epos.long()
        r = r + e.float()[rows].sum(1)
    return r


def qkv_heads(qkv: torch.Tensor, bias, pos: torch.Tensor, cos, sin, L, v_first, lam):
    """fp32 (q, k, v) of packed projection rows: + bias, neighbours-paired rotation of the first
    rot_dims dimensions, per-head RMS norm of q and k, value mixing."""
    T = qkv.shape[0]
    dk, dv = L.pads
    x = qkv.float() if bias is None else qkv.float() + bias
    nq, nk = L.heads * dk, L.kv_heads * dk
    q, k = x[:, :nq].reshape(T, L.heads, dk), x[:, nq:nq + nk].reshape(T, L.kv_heads, dk)
    v = x[:, nq + nk:nq + nk + L.kv_heads * dv].reshape(T, L.kv_heads, dv)

    def turn(t):
        if cos is None or L.rot_dims < 2:
            return t
        n = L.rot_dims // 2
        c, s = cos[pos][:, None, :n], sin[pos][:, None, :n]
        a, b = t[..., 0:2 * n:2], t[..., 1:2 * n:2]
        r = t.clone()
        r[..., 0:2 * n:2], r[..., 1:2 * n:2] = a * c - b * s, b * c + a * s
        return r

    def unit(t):
        return t * torch.rsqrt(t.pow(2).sum(-1, keepdim=True) / L.dim + L.eps) if L.norm else t

    q, k = unit(turn(q)), unit(turn(k))
    if v_first is not None:
        v = (1 - lam) * v + lam * v_first.float()
    return q, k, v


def cache_rows(k_cache: torch.Tensor, v_cache: torch.Tensor, k: torch.Tensor, v: torch.Tensor, slots: torch.Tensor) -> None:
    """Write k / v [T, G, d] to a token-row paged cache [pages, G, P, d]."""
    P = k_cache.shape[2]
    ok = slots >= 0
    pg, off = slots[ok] // P, slots[ok] % P
    k_cache[pg, :, off] = k[ok].to(k_cache.dtype)
    v_cache[pg, :, off] = v[ok].to(v_cache.dtype)


def attn_decode_rows(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, block_tables: torch.Tensor,
                     seq_lens: torch.Tensor, scale: float, window: int = 0) -> torch.Tensor:
    """One query token per sequence over a token-row paged cache; keys and values of any size
    (``window``: the last that many tokens only)."""
    B, Hq, _ = q.shape
    Hkv, P = k_cache.shape[1], k_cache.shape[2]
    out = torch.zeros(B, Hq, v_cache.shape[3], dtype=q.dtype, device=q.device)
    for b in range(B):
        n = int(seq_lens[b])
        if n == 0:
            continue
        pages = block_tables[b, :(n + P - 1) // P].long()
        k = k_cache[pages].permute(1, 0, 2, 3).reshape(Hkv, -1, k_cache.shape[3])[:, :n].float()
        v = v_cache[pages].permute(1, 0, 2, 3).reshape(Hkv, -1, v_cache.shape[3])[:, :n].float()
        a = max(0, n - window) if window else 0
        k, v = k[:, a:], v[:, a:]
        s = torch.matmul(q[b].float().view(Hkv, Hq // Hkv, -1), k.transpose(1, 2)) * scale
        out[b] = torch.matmul(torch.softmax(s, -1), v).reshape(Hq, -1).to(q.dtype)
    return out


def rms_rows(x: torch.Tensor, w: torch.Tensor, width: int, eps: float) -> torch.Tensor:
    """Weighted RMS norm of zero-padded rows whose true width is ``width``; fp32."""
    x = x.float()
    return x * torch.rsqrt(x.pow(2).sum(-1, keepdim=True) / width + eps) * w


def conv_heads(x: torch.Tensor, pos: torch.Tensor, L, conv: torch.Tensor, qw: torch.Tensor, kw: torch.Tensor, tails,
               slots: torch.Tensor, edges, P: int):
    """fp32 (q, k, v, gate) of packed q | k | gate rows; ``tails`` (the last projected rows of every page's
    tokens, entry position % (taps - 1)) is read before and written after."""
    dk, dv = L.pads
    H, G, R = L.heads, L.kv_heads, conv.shape[0] - 1
    C = (H + G) * dk
    u, conv, qw, kw = x[:, :C].float(), conv.float(), qw.float(), kw.float()
    y = torch.zeros_like(u)
    T = u.shape[0]
    start, pages, ends = list(range(T)), [-1] * T, list(range(1, T + 1))
    if edges.block_tables is None:
        t = 0
        for s, n in enumerate(edges.lens):
            pg = -1 if edges.prev_pages is None else int(edges.prev_pages[s])
            start[t:t + n], pages[t:t + n], ends[t:t + n] = [t] * n, [pg] * n, [t + n] * n
            t += n
    for t in range(T):
        p = int(pos[t])
        for d in range(min(R, p) + 1):
            if t - d >= start[t]:
                v = u[t - d]
            else:
                pg = pages[t] if edges.block_tables is None else int(edges.block_tables[t, (p - d) // P])
                if pg < 0:
                    continue
                v = tails[pg, (p - d) % R].float()
            y[t] += conv[R - d] * v
    for t in range(T):
        if R and int(slots[t]) >= 0 and t + R >= ends[t]:
            tails[int(slots[t]) // P, int(pos[t]) % R] = u[t].to(tails.dtype)
    q, k = y[:, :H * dk].view(T, H, dk), y[:, H * dk:].view(T, G, dk)
    v = torch.zeros(T, G, dv)
    v[..., :dk] = k
    return rms_rows(q, qw, L.dim, L.eps), rms_rows(k, kw, L.dim, L.eps), v, torch.sigmoid(x[:, C:C + H].float())


def rotate_heads(x: torch.Tensor, pos: torch.Tensor, rot: tuple, at: int, dims: int) -> torch.Tensor:
    """fp32 x [T, H, d] with columns at .. at + dims rotated, i paired with i + dims / 2."""
    y, n = x.float().clone(), dims // 2
    c, s = rot[0][pos][:, None, :n], rot[1][pos][:, None, :n]
    a, b = x[..., at:at + n].float(), x[..., at + n:at + 2 * n].float()
    y[..., at:at + n], y[..., at + n:at + 2 * n] = a * c - b * s, b * c + a * s
    return y


def latent_rows(x: torch.Tensor, pos: torch.Tensor, rot: tuple, L, dtype, qw, cw, cache, slots):
    T = x.shape[0]
    cq = rms_rows(x[:, :L.qp], qw, L.q_rank, L.eps).to(dtype)
    at, lat = L.qp, None
    if L.own:
        lat = torch.zeros(T, L.ck, dtype=dtype)
        lat[:, :L.rp] = rms_rows(x[:, at:at + L.rp], cw, L.kv_rank, L.eps).to(dtype)
        at += L.rp
        lat[:, L.rp:L.rp + L.rot] = rotate_heads(x[:, None, at:at + L.rot], pos, rot, 0, L.rot)[:, 0].to(dtype)
        at += L.rotp
        P, ok = cache.shape[2], slots >= 0
        cache[slots[ok] // P, 0, slots[ok] % P] = lat[ok]
    return cq, torch.sigmoid(x[:, at:at + L.heads].float()), lat


def head_gemm(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """y[m, h] = x[m, h] w[h]^T."""
    return torch.matmul(x.float().transpose(0, 1), w.float().transpose(1, 2)).transpose(0, 1).to(x.dtype)


def route(h: torch.Tensor, wr: torch.Tensor, experts: int, top: int, gated: bool):
    z = h.float() @ wr.float().t()
    v, i = torch.topk(z[:, :experts], top, dim=-1)
    return i.to(torch.int32), torch.sigmoid(v), z[:, experts].contiguous() if gated else None


def experts(h: torch.Tensor, ids: torch.Tensor, wt: torch.Tensor, wgu: torch.Tensor, wd: torch.Tensor) -> torch.Tensor:
    """Row t * top + k: expert ids[t, k] on wt[t, k] * h[t] (gate | up interleaved in 64-row blocks)."""
    T, top = ids.shape
    y = torch.zeros(T * top, wd.shape[1], dtype=h.dtype)
    flat, xs = ids.reshape(-1), h.float().repeat_interleave(top, 0) * wt.reshape(-1, 1)
    for e in flat.unique().tolist():
        r = flat == e
        gu = (xs[r] @ wgu[e].float().t()).to(h.dtype)
        y[r] = (silu_mul(gu, 64).float() @ wd[e].float().t()).to(h.dtype)
    return y
