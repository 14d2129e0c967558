"""The general decoder ops (streams, QKV heads, short-convolution heads, any-head-size, windowed and
latent attention, routed experts, fp32 products), each alone, against plain fp64 formulas: the CPU references and the GPU kernels."""
import pytest
import torch

import relurax_oracle as R
import sufolix_oracle as O
from operator_amd import ops
from operator_amd.ops import decoder as dec

DEV = "cpu"


@pytest.fixture(autouse=True, params=["cpu", pytest.param("cuda", marks=pytest.mark.gpu)])
def device(request):
    global DEV
    DEV = request.param
    return DEV


def _g(seed):
    return torch.Generator().manual_seed(seed)


def _rand(g, *shape, scale=1.0):
    return torch.randn(*shape, generator=g) * scale


def _close(got, want, tol):
    got, want = got.double().cpu(), want.double().cpu()
    err = (got - want).abs().max().item()
    assert torch.isfinite(got).all()
    assert err <= tol * max(1.0, want.abs().max().item()), (err, want.abs().max().item())


# ---------------------------------------------------------------- streams
@pytest.mark.parametrize("S,width,ld", [(1, 192, 192), (2, 200, 256), (3, 1000, 1024), (4, 4096, 4096), (5, 130, 192),
                                        (8, 2500, 2560)])
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_stream_step(S, width, ld, dtype):
    g = _g(S * 100 + width)
    T, V, top, eps = 5, 37, 2, 1e-5
    pad = torch.zeros(ld)
    pad[:width] = 1
    table = (_rand(g, V, ld) * pad).to(dtype)
    ids = torch.tensor([3, 0, 36, 5, 3])
    inp, out, mix = _rand(g, S), _rand(g, S), _rand(g, S, S)
    w = (1 + 0.1 * _rand(g, ld)) * pad
    c = lambda t: t.to(DEV)  # noqa: E731
    x, h = dec.stream_init(c(ids), c(table), 3.5, S, width, c(inp), c(w), eps)
    xr = (table[ids].double() * 3.5)[:, None].repeat(1, S, 1)
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    _close(x, xr, 1e-6)
    norm = lambda u: (u / torch.sqrt((u * u).sum(-1, keepdim=True) / width + eps)) * w.double()  # noqa: E731
    _close(h, norm(torch.einsum("tsw,s->tw", xr, inp.double())), tol)
    # a middle step: gated rows + routed rows through a position table
    xr = _rand(g, T, S, ld).double() * pad
    y, e = (_rand(g, T, ld) * pad).to(dtype), (_rand(g, 16, ld) * pad).to(dtype)
    gate = _rand(g, T)
    pos = torch.randint(0, 16, (T, top), generator=g).to(torch.int32)
    yr = torch.sigmoid(gate.double())[:, None] * y.double() + e.double()[pos.long()].sum(1)
    x = c(xr.float())
    h = dec.stream_step(x, dec.SublayerOut(c(y), c(gate), c(e), c(pos), top), dec.Stream(c(inp), c(mix), c(out)), c(inp),
                        c(w), width, eps, dtype)
    xn = torch.einsum("tsw,sr->trw", xr, mix.double()) + out.double()[None, :, None] * yr[:, None]
    _close(x, xn, 1e-5)
    _close(h, norm(torch.einsum("tsw,s->tw", xn, inp.double())), tol)
    # fp32 slabs and identity routing rows; the last step picks rows and keeps the streams
    slabs = _rand(g, 3, T, ld) * pad
    e = (_rand(g, T * top, ld) * pad).to(dtype)
    sk = slabs.sum(0) if DEV == "cpu" else ops.SplitK(c(slabs).reshape(-1), 3, T, ld)   # split-K is the GPU's
    rows = torch.tensor([4, 1])
    x = c(xr.float())
    h = dec.stream_step(x, dec.SublayerOut(sk, None, c(e), None, top), dec.Stream(c(inp), c(mix), c(out)), None, c(w),
                        width, eps, dtype, rows=c(rows), write_x=False)
    yr = slabs.double().sum(0) + e.double().view(T, top, ld).sum(1)
    xn = torch.einsum("tsw,sr->trw", xr, mix.double()) + out.double()[None, :, None] * yr[:, None]
    _close(h, norm(xn.sum(1))[rows], tol)
    _close(x, xr, 1e-6)


# ---------------------------------------------------------------- QKV heads
LAYOUTS = [(10, 2, 56, 40, 24), (6, 3, 40, 24, 32), (4, 4, 128, 128, 128), (5, 1, 96, 64, 20), (2, 1, 16, 40, 16),
           (3, 3, 200, 160, 100), (16, 1, 64, 96, 2)]


def _cache_rows(cache, kind, dtype):
    """Token-row view [pages, G, P, d] of a layer's cache (bf16 GPU caches are tiled)."""
    c = cache.cpu()
    if dtype == torch.float32 or DEV == "cpu":
        return c
    n, G, P, d = c.shape
    t = c.reshape(n, G, P // 16, 16 * d)
    if kind == "k":
        return t.view(n, G, P // 16, d // 8, 16, 8).permute(0, 1, 2, 4, 3, 5).reshape(n, G, P, d)
    return t.view(n, G, P // 16, d // 32, 4, 16, 2, 4).permute(0, 1, 2, 4, 7, 3, 6, 5).reshape(n, G, P, d)


@pytest.mark.parametrize("H,G,D,Dv,rot", LAYOUTS)
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("slabs", [0, 3])
def test_qkv_heads(H, G, D, Dv, rot, dtype, slabs):
    g = _g(H * D + Dv)
    L = dec.HeadLayout(H, G, D, Dv, rot, True, 1e-5)
    dk, dv = L.pads
    T, P, pages = 7, 32, 4
    real = torch.zeros(L.ncol)
    for h in range(H + G):
        real[h * dk:h * dk + D] = 1
    for h in range(G):
        real[(H + G) * dk + h * dv:(H + G) * dk + h * dv + Dv] = 1
    if slabs:
        sl = _rand(g, slabs, T, L.ncol) * real
        src = sl.sum(0) if DEV == "cpu" else ops.SplitK(sl.reshape(-1).to(DEV), slabs, T, L.ncol)
        rows = sl.double().sum(0)
    else:
        r = (_rand(g, T, L.ncol) * real).to(dtype)
        src, rows = r.to(DEV), r.double()
    bias = _rand(g, L.ncol) * real
    pos = torch.tensor([0, 1, 2, 15, 16, 500, 999])
    slots = torch.tensor([0, 17, 31, 64 + 15, -1, 64 + 16, 127])
    vf = _rand(g, T, G, dv).to(dtype)
    lam = torch.tensor([0.3])
    tabs = dec.rotary_tables(1000, 30000.0, rot, device=DEV)
    kc = torch.zeros(pages, G, P, dk, dtype=dtype, device=DEV)
    vc = torch.zeros(pages, G, P, dv, dtype=dtype, device=DEV)
    c = lambda t: t.to(DEV)  # noqa: E731
    q, k, v = dec.qkv_heads(src, c(pos), tabs, L, dtype, bias=c(bias), cache=(kc, vc), slots=c(slots), v_first=c(vf), lam=c(lam))
    x = rows + bias.double()
    qr = x[:, :H * dk].view(T, H, dk)[..., :D]
    kr = x[:, H * dk:(H + G) * dk].view(T, G, dk)[..., :D]
    vr = x[:, (H + G) * dk:(H + G) * dk + G * dv].view(T, G, dv)
    qr = O.rms(O.rotate(qr, pos.tolist(), 30000.0, rot), 1e-5)
    kr = O.rms(O.rotate(kr, pos.tolist(), 30000.0, rot), 1e-5)
    vr = O.mix_values(vr, vf.double(), 0.3)
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    _close(q[..., :D], qr, tol)
    _close(k[..., :D], kr, tol)
    _close(v[..., :Dv], vr[..., :Dv], tol)
    assert q[..., D:].abs().max().item() == 0 if dk > D else True
    kl, vl = _cache_rows(kc, "k", dtype), _cache_rows(vc, "v", dtype)
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            assert torch.equal(kl[s // P, :, s % P], k[t].cpu()) and torch.equal(vl[s // P, :, s % P], v[t].cpu())
    used = torch.zeros(pages * P, dtype=torch.bool)
    used[slots[slots >= 0]] = True
    assert kl.permute(0, 2, 1, 3).reshape(pages * P, -1)[~used].abs().max().item() == 0
    assert vl.permute(0, 2, 1, 3).reshape(pages * P, -1)[~used].abs().max().item() == 0


# ---------------------------------------------------------------- attention
def _padded(t, d):
    o = torch.zeros(*t.shape[:-1], d, dtype=t.dtype)
    o[..., :t.shape[-1]] = t
    return o


def _spiky(g, T, H, G, D, Dv, dtype):
    """q, k, v where a few far keys stand out for a few queries."""
    q, k, v = _rand(g, T, H, D), _rand(g, T, G, D), _rand(g, T, G, Dv)
    for t, j in ((T - 1, 0), (T - 1, T // 2), (T // 2, min(1, T - 1)), (T // 3, T // 3)):
        q[t] *= 2.0
        k[j] = q[t, :1] * 1.5   # every kv head
    return q.to(dtype), k.to(dtype), v.to(dtype)


SHAPES = [(10, 2, 56, 40), (6, 3, 40, 24), (4, 4, 128, 128), (5, 1, 96, 64), (2, 1, 16, 40), (3, 3, 200, 160),
          (16, 1, 64, 96), (34, 2, 32, 32), (12, 4, 80, 100), (7, 7, 256, 256)]


@pytest.mark.parametrize("H,G,D,Dv", SHAPES)
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_attn_prefill(H, G, D, Dv, dtype):
    g = _g(H + D)
    L = dec.HeadLayout(H, G, D, Dv)
    dk, dv = L.pads
    lens = [1, 63, 64, 65, 131, 300]
    parts = [_spiky(g, n, H, G, D, Dv, dtype) for n in lens]
    q, k, v = (torch.cat([_padded(p[i], d) for p in parts]).to(DEV) for i, d in ((0, dk), (1, dk), (2, dv)))
    scale = 0.7 / D ** 0.5
    o = dec.attn_gd_prefill(q, k, v, lens, L, scale)
    a = 0
    for n, (pq, pk, pv) in zip(lens, parts):
        want = O.attend(pq.double(), pk.double(), pv.double(), scale)
        got = o[a:a + n, :H * dv].view(n, H, dv)
        _close(got[..., :Dv], want, 3e-5 if dtype == torch.float32 else 1.5e-2)
        a += n
    assert L.ocol == H * dv or o[:, H * dv:].abs().max().item() == 0
    # a shared prefix of 37 keys before sequence 1 and 4 only
    pre = _spiky(g, 37, H, G, D, Dv, dtype)
    pfx = [0, 37, 0, 0, 21, 0]
    o = dec.attn_gd_prefill(q, k, v, lens, L, scale, work=_work(lens, DEV),
                            prefix=(_padded(pre[1], dk).to(DEV), _padded(pre[2], dv).to(DEV),
                                    torch.tensor(pfx, dtype=torch.int32, device=DEV), pfx))
    a = 0
    for n, n0, (pq, pk, pv) in zip(lens, pfx, parts):
        want = O.attend(torch.cat([pre[0][:n0], pq]).double(), torch.cat([pre[1][:n0], pk]).double(),
                        torch.cat([pre[2][:n0], pv]).double(), scale)[n0:]
        _close(o[a:a + n, :H * dv].view(n, H, dv)[..., :Dv], want, 3e-5 if dtype == torch.float32 else 1.5e-2)
        a += n


def _work(lens, dev):
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    ws, wq = ops.prefill_work_list(lens, dec.GD_BLOCK_Q)
    return tuple(torch.tensor(t, dtype=torch.int32, device=dev) for t in (cu, ws, wq)) + (dec.GD_VARIANT,)


@pytest.mark.parametrize("H,G,D,Dv", SHAPES)
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("page", [16, 64])
def test_attn_decode(H, G, D, Dv, dtype, page):
    g = _g(H + D)
    L = dec.HeadLayout(H, G, D, Dv, 0, False)
    dk, dv = L.pads
    lens = [1, 15, 16, 17, 33, 128, 129, 700, 0]
    B, mp = len(lens), -(-704 // page)
    total = sum(-(-n // page) for n in lens)
    perm = torch.randperm(total + 3, generator=g)   # pages in no order, some foreign
    kc = torch.full((total + 3, G, page, dk), 7.0, dtype=dtype, device=DEV)   # stale rows: finite junk
    vc = torch.full((total + 3, G, page, dv), float("inf") if dtype == torch.bfloat16 else 9.0, dtype=dtype, device=DEV)
    bt = torch.zeros(B, mp, dtype=torch.int32)
    seqs, at = [], 0
    tabs = None
    for b, n in enumerate(lens):
        q, k, v = _spiky(g, max(n, 1), H, G, D, Dv, dtype)
        seqs.append((q, k, v))
        npg = -(-n // page)
        pages = perm[at:at + npg]
        at += npg
        bt[b, :npg] = pages.to(torch.int32)
        if n == 0:
            continue
        rows = torch.zeros(n, L.ncol)
        rows[:, H * dk:(H + G) * dk] = _padded(k.float(), dk).reshape(n, -1)
        rows[:, (H + G) * dk:(H + G) * dk + G * dv] = _padded(v.float(), dv).reshape(n, -1)
        slots = torch.tensor([int(pages[j // page]) * page + j % page for j in range(n)])
        dec.qkv_heads(rows.to(dtype).to(DEV), torch.arange(n, device=DEV), tabs, L, dtype, cache=(kc, vc), slots=slots.to(DEV))
    q = torch.stack([_padded(s[0][-1], dk) for s in seqs]).to(DEV)
    scale = 0.7 / D ** 0.5
    for splits in (1, 2, 4):
        o = dec.attn_gd_decode(q, (kc, vc), bt.to(DEV), torch.tensor(lens, dtype=torch.int32, device=DEV), L, scale, splits)
        for b, n in enumerate(lens):
            got = o[b, :H * dv].view(H, dv)[:, :Dv]
            if n == 0:
                assert got.abs().max().item() == 0
                continue
            want = O.attend(*(t.double() for t in seqs[b]), scale)[-1]
            _close(got, want, 3e-5 if dtype == torch.float32 else 1.5e-2)


# ---------------------------------------------------------------- experts
def _expert_weights(g, E, ff, ld, dtype):
    gate, up = _rand(g, E, ff, ld, scale=ld ** -0.5), _rand(g, E, ff, ld, scale=ld ** -0.5)
    down = _rand(g, E, ld, ff, scale=ff ** -0.5)
    gate, up, down = gate.to(dtype), up.to(dtype), down.to(dtype)
    wgu = torch.stack([ops.interleave_gate_up(a, b) for a, b in zip(gate, up)])
    return gate, up, down, wgu


@pytest.mark.parametrize("T,E,top,ff,ld", [(1, 4, 1, 128, 128), (16, 8, 2, 192, 256), (33, 5, 5, 128, 192), (70, 3, 2, 128, 320),
                                           (300, 4, 2, 256, 256), (2100, 6, 3, 128, 128), (64, 200, 4, 128, 128)])
@pytest.mark.parametrize("dtype,plan", [(torch.bfloat16, p) for p in (None, 0, 64, 128, 256)] + [(torch.float32, None)])
def test_route_and_experts(T, E, top, ff, ld, dtype, plan):
    if plan == 0 and T * top > dec.MOE_LIST_MAX_SLOTS:
        pytest.skip("more rows than an expert's list holds")
    if DEV == "cpu" and (plan is not None or T > 300):
        pytest.skip("kernel choice and tile borders are the GPU's")
    g = _g(T + E)
    gate, up, down, wgu = _expert_weights(g, E, ff, ld, dtype)
    h = _rand(g, T, ld).to(dtype)
    wr = torch.zeros(dec.router_rows(E), ld)
    wr[:E + 1] = _rand(g, E + 1, ld, scale=ld ** -0.5) * 2
    wr = wr.to(dtype)
    ids, wt, gt = dec.route(h.to(DEV), wr.to(DEV), E, top, True)
    z = h.double() @ wr.double().T
    val, idx = torch.topk(z[:, :E], top)
    close = torch.topk(z[:, :E], min(E, top + 1))[0]
    sure = torch.ones(T, dtype=torch.bool) if top == E else (close[:, top - 1] - close[:, top]) > 1e-3
    assert sure.float().mean() > 0.8
    i = ids.cpu().long()
    assert torch.equal(i.sort(1)[0][sure], idx.sort(1)[0][sure]) and int(i.min()) >= 0 and int(i.max()) < E
    _close(wt, torch.sigmoid(z.gather(1, i)), 1e-4)
    _close(gt, z[:, E], 1e-4)
    rows, pos = dec.experts(h.to(DEV), ids, wt, wgu.to(DEV), down.to(DEV), plan)
    p = torch.arange(T * top).view(T, top) if pos is None else pos.cpu().long()
    got = rows.double().cpu()[p].sum(1)
    w = wt.cpu().double()
    want = torch.zeros(T, ld, dtype=torch.float64)
    for e in range(E):
        for k in range(top):
            t = (i[:, k] == e).nonzero().flatten()
            if len(t):
                x = w[t, k, None] * h[t].double()
                a, b = x @ gate[e].double().T, x @ up[e].double().T
                want[t] += (a * torch.sigmoid(a) * b) @ down[e].double().T
    _close(got, want, 2e-5 if dtype == torch.float32 else 2e-2)


def test_experts_all_tokens_to_one():
    """One expert takes everything (its segment spans many tiles), the others stay empty."""
    g = _g(3)
    E, ff, ld = 6, 128, 256
    gate, up, down, wgu = _expert_weights(g, E, ff, ld, torch.bfloat16)
    for T, plan in ((40, 0), (40, 64), (200, 128), (1100, 256)):
        h = _rand(g, T, ld).to(torch.bfloat16)
        ids = torch.full((T, 1), 4, dtype=torch.int32, device=DEV)
        wt = torch.full((T, 1), 0.5, device=DEV)
        rows, pos = dec.experts(h.to(DEV), ids, wt, wgu.to(DEV), down.to(DEV), plan)
        p = torch.arange(T) if pos is None else pos.cpu().long().flatten()
        x = 0.5 * h.double()
        a, b = x @ gate[4].double().T, x @ up[4].double().T
        _close(rows.double().cpu()[p], (a * torch.sigmoid(a) * b) @ down[4].double().T, 2e-2)


def test_router_survives_nan_rows():
    """Padding rows of a captured batch can hold anything; their expert ids must stay in range."""
    h = torch.full((17, 128), float("nan"), dtype=torch.bfloat16, device=DEV)
    h[3] = 1
    ids, _, _ = dec.route(h, torch.randn(16, 128, device=DEV).to(torch.bfloat16), 12, 3, False)
    assert int(ids.min()) >= 0 and int(ids.max()) < 12


@pytest.mark.parametrize("M,N,K", [(1, 64, 64), (65, 192, 128), (200, 1000, 320)])
def test_gemm_f32(M, N, K):
    g = _g(M)
    x, w = _rand(g, M, K), _rand(g, N, K)
    y = ops.linear(x.to(DEV), w.to(DEV))
    _close(y, x.double() @ w.double().T, 2e-6 * K ** 0.5)
    if N % 64 == 0:
        gu = ops.interleave_gate_up(w, w.flip(0).contiguous())
        y = ops.gate_up_silu(x.to(DEV), gu.to(DEV), 64)
        a, b = x.double() @ w.double().T, x.double() @ w.flip(0).double().T
        _close(y, a * torch.sigmoid(a) * b, 2e-6 * K ** 0.5)


@pytest.mark.parametrize("M,N,K", [(64, 256, 512), (128, 1024, 256), (256, 512, 1024), (192, 128, 256)])
def test_narrow_gate_up_splits_k(M, N, K):
    g = _g(M)
    a, b, x = (_rand(g, *s, scale=K ** -0.25).to(torch.bfloat16) for s in ((N // 2, K), (N // 2, K), (M, K)))
    assert ops._gu_splits(M, N, K) > 1
    y = ops.gate_up_silu(x.to(DEV), ops.interleave_gate_up(a, b).to(DEV), 64)
    u, v = x.double() @ a.double().T, x.double() @ b.double().T
    _close(y, u * torch.sigmoid(u) * v, 2e-2)


# ---------------------------------------------------------------- norms of outputs, gated activations
@pytest.mark.parametrize("T,width,ld", [(1, 200, 256), (5, 4096, 4096), (600, 1000, 1024), (3, 9000, 9024)])
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_stream_step_with_output_norm(T, width, ld, dtype):
    """x + norm(y), from rows and from fp32 slabs, and the next norm of the sum."""
    g = _g(T + width)
    pad = torch.zeros(ld)
    pad[:width] = 1
    x0, y = _rand(g, T, 1, ld) * pad, (3 * _rand(g, T, ld) * pad).to(dtype)
    w, pw = (1 + 0.1 * _rand(g, ld)) * pad, (1 + 0.3 * _rand(g, ld)) * pad
    one = torch.ones(1, device=DEV)
    hc = dec.Stream(one, one.view(1, 1), one)
    norm = lambda u, q: u / torch.sqrt((u * u).sum(-1, keepdim=True) / width + 1e-5) * q.double()  # noqa: E731
    slabs = _rand(g, 3, T, ld) * pad
    for src, yr in ((y.to(DEV), y.double()),
                    (slabs.sum(0) if DEV == "cpu" else ops.SplitK(slabs.reshape(-1).to(DEV), 3, T, ld), slabs.double().sum(0))):
        x = x0.clone().to(DEV)
        h = dec.stream_step(x, dec.SublayerOut(src), hc, one, w.to(DEV), width, 1e-5, dtype, post_w=pw.to(DEV))
        xn = x0.double()[:, 0] + norm(yr, pw)
        _close(x[:, 0], xn, 2e-6)
        _close(h, norm(xn, w), 1e-5 if dtype == torch.float32 else 1e-2)
    x = x0.clone().to(DEV)
    rows = torch.tensor([T - 1, 0], device=DEV)
    h = dec.stream_step(x, dec.SublayerOut(y.to(DEV)), hc, None, w.to(DEV), width, 1e-5, dtype, rows=rows, write_x=False, post_w=pw.to(DEV))
    xn = x0.double()[:, 0] + norm(y.double(), pw)
    _close(h, norm(xn, w)[[T - 1, 0]], 1e-5 if dtype == torch.float32 else 1e-2)
    assert torch.equal(x.cpu(), x0)


@pytest.mark.parametrize("M", [1, 9, 32, 64, 128, 192, 256, 300])
@pytest.mark.parametrize("ff,K", [(128, 128), (192, 320), (1024, 1024)])
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("act", [ops.SILU, ops.GELU_TANH])
def test_gated_activations(M, ff, K, dtype, act):
    g = _g(M + ff)
    x, gate, up = _rand(g, M, K).to(dtype), (3 * _rand(g, ff, K, scale=K ** -0.5)).to(dtype), _rand(g, ff, K, scale=K ** -0.5).to(dtype)
    y = ops.gate_up_silu(x.to(DEV), ops.interleave_gate_up(gate, up).to(DEV), ops.GU_BLOCK, act)
    a, b = x.double() @ gate.double().T, x.double() @ up.double().T
    _close(y, (R.gelu_tanh(a) if act == ops.GELU_TANH else a * torch.sigmoid(a)) * b, 1e-5 if dtype == torch.float32 else 1.5e-2)


def test_gelu_on_the_tuned_decode_shapes():
    """The widest gate | up projections have kernels of their own."""
    if DEV == "cpu":
        pytest.skip("kernel choice is the GPU's")
    g = torch.Generator(device=DEV).manual_seed(1)
    w = torch.randn(28672, 4096, generator=g, device=DEV, dtype=torch.bfloat16) / 32
    for M in (16, 64, 128, 256):
        x = torch.randn(M, 4096, generator=g, device=DEV, dtype=torch.bfloat16)
        y = ops.gate_up_silu(x, w, ops.GU_BLOCK, ops.GELU_TANH)
        z = (x.float() @ w.float().t()).view(M, 224, 2, 64)
        want = torch.nn.functional.gelu(z[:, :, 0], approximate="tanh") * z[:, :, 1]
        _close(y, want.reshape(M, -1), 1e-2)


# ---------------------------------------------------------------- heads behind short convolutions
@pytest.mark.parametrize("H,G,D", [(4, 2, 24), (6, 1, 64), (3, 3, 100), (8, 4, 128), (2, 1, 250)])
@pytest.mark.parametrize("taps", [1, 2, 4, 7])
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_conv_heads(H, G, D, taps, dtype):
    """Packed prompts, one of them behind tokens of an earlier page, then decode steps from the pages."""
    g = _g(H * D + taps)
    L = dec.HeadLayout(H, G, D, D, eps=1e-5)
    (dk, dv), P, pages, n = L.pads, 16, 12, dec.conv_ncol(L)
    C = (H + G) * dk
    lens, skip, more = [1, 2, 37, 5, 20], [0, 0, 0, 16, 0], 19
    owned = [[3, 9], [1, 6], [0, 2, 8, 10], [5, 7, 4], [11, 3]]   # pages of every sequence (the last one takes over a page)
    total = [a + b + more for a, b in zip(lens, skip)]
    real = torch.zeros(n)
    for h in range(H + G):
        real[h * dk:h * dk + D] = 1
    real[C:C + H] = 1
    seqs = [(_rand(g, t, n) * real).to(dtype) for t in total]
    conv = torch.zeros(taps, C)
    conv[:, real[:C] > 0] = _rand(g, taps, int(real[:C].sum()))
    qw, kw = torch.zeros(dk), torch.zeros(dk)
    qw[:D], kw[:D] = 1 + 0.2 * _rand(g, D), 1 + 0.2 * _rand(g, D)
    conv, qw, kw = (t.to(dtype).to(DEV) for t in (conv, qw, kw))
    cut = lambda x, a, b: x[:, a * dk:b * dk].reshape(len(x), b - a, dk)[..., :D].double()  # noqa: E731

    def want(s):
        x = seqs[s]
        c = R.short_conv(x[:, :C].double(), conv.double().cpu().T)
        q, k = cut(c, 0, H), cut(c, H, H + G)
        return R.rms(q, 1e-5, qw[:D].double().cpu()), R.rms(k, 1e-5, kw[:D].double().cpu()), k, torch.sigmoid(x[:, C:C + H].double())

    kc, vc = (torch.full((pages, G, P, d), 5.0, dtype=dtype, device=DEV) for d in (dk, dv))
    tails = torch.full((pages, taps - 1, C), 5.0, dtype=dtype, device=DEV) if taps > 1 else None
    slot = lambda s, t: owned[s][t // P] * P + t % P  # noqa: E731
    tol = 2e-5 if dtype == torch.float32 else 1.5e-2

    def prefill(which, start, lens, prev):
        x = torch.cat([seqs[s][a:a + m] for s, a, m in zip(which, start, lens)]).to(DEV)
        pos = torch.cat([torch.arange(a, a + m) for a, m in zip(start, lens)])
        slots = torch.tensor([slot(s, t) for s, a, m in zip(which, start, lens) for t in range(a, a + m)])
        cu = torch.tensor([0] + torch.tensor(lens).cumsum(0).tolist(), dtype=torch.int32, device=DEV)
        e = dec.SequenceEdges(cu, lens, None if prev is None else torch.tensor(prev, dtype=torch.int32, device=DEV))
        out = dec.conv_heads(x, pos.to(DEV), L, dtype, conv, qw, kw, (kc, vc), tails, slots.to(DEV), e)
        at = 0
        for s, a, m in zip(which, start, lens):
            for got, ref, d in zip(out, want(s), (D, D, D, H)):
                _close(got[at:at + m][..., :d], ref[a:a + m], tol)
            at += m

    prefill([3, 0], [0, 0], [16, 1], None)   # a shared head, and a sequence that ends
    live = [1, 2, 3, 4]                      # the last one takes over a page of the one that ended
    prefill(live, skip[1:], lens[1:], [-1, -1, owned[3][0], -1])
    at = {s: skip[s] + lens[s] for s in live}
    for step in range(more if DEV == "cuda" else 4):
        live = [s for s in live if slot_ok(owned[s], at[s], P)]
        x = torch.stack([seqs[s][at[s]] for s in live] + [torch.zeros(n, dtype=dtype)]).to(DEV)   # a padding row
        if step % 2 and DEV == "cuda":
            x = ops.SplitK(torch.cat([0.25 * x.float(), 0.75 * x.float()]).reshape(-1), 2, *x.shape)
        pos = torch.tensor([at[s] for s in live] + [0])
        slots = torch.tensor([slot(s, at[s]) for s in live] + [-1])
        bt = torch.zeros(len(live) + 1, 5, dtype=torch.int32)
        for i, s in enumerate(live):
            bt[i, :len(owned[s])] = torch.tensor(owned[s])
        out = dec.conv_heads(x, pos.to(DEV), L, dtype, conv, qw, kw, (kc, vc), tails, slots.to(DEV), dec.SequenceEdges(block_tables=bt.to(DEV)))
        for i, s in enumerate(live):
            ref = want(s)
            _close(out[0][i, :, :D], ref[0][at[s]], tol)
            _close(out[3][i], ref[3][at[s]], tol)
            at[s] += 1
    kl, vl = _cache_rows(kc, "k", dtype), _cache_rows(vc, "v", dtype)
    for s in live:
        ref = want(s)
        for t in range(at[s]):
            pg, off = owned[s][t // P], t % P
            _close(kl[pg, :, off, :D], ref[1][t], tol)
            _close(vl[pg, :, off, :D], ref[2][t], tol)
            assert vl[pg, :, off, D:].abs().sum().item() == 0


def slot_ok(pages, t, P):
    return t < len(pages) * P


# ---------------------------------------------------------------- windows and head gates
@pytest.mark.parametrize("H,G,D", [(4, 2, 24), (8, 8, 64), (16, 1, 128), (6, 2, 200)])
@pytest.mark.parametrize("window", [1, 15, 64, 65, 130, 1000])
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_windowed_attention(H, G, D, window, dtype):
    """Every query's last visible and first hidden key stand out (prefill, behind a prefix, and decode)."""
    g = _g(H + D + window)
    L = dec.HeadLayout(H, G, D, D)
    dk, dv = L.pads
    lens = [1, 64, 65, 290]
    q, k, v = ([_rand(g, n, h, D).to(dtype) for n in lens] for h in (H, G, G))
    for n, a, b in zip(lens, q, k):   # keys at both sides of some queries' edge
        for t in range(window, n, 37):
            b[t - window] = a[t, :1] * 1.5
            b[t - window + 1] = a[t, :1]
    gate = torch.sigmoid(_rand(g, sum(lens), H))
    scale, tol = 0.7 / D ** 0.5, 3e-5 if dtype == torch.float32 else 1.5e-2
    pack = lambda x, d: torch.cat([_padded(t, d) for t in x]).to(DEV)  # noqa: E731
    o = dec.attn_gd_prefill(pack(q, dk), pack(k, dk), pack(v, dv), lens, L, scale, window=window, gate=gate.to(DEV))
    full = [R.attend(a.double(), b.double(), c.double(), scale, window) for a, b, c in zip(q, k, v)]
    got = o[:, :H * dv].view(-1, H, dv)[..., :D]
    _close(got, torch.cat(full) * gate.double()[..., None], tol)
    # the last sequence again, its first 70 tokens as a shared prefix
    pl, n = 70, lens[3]
    o = dec.attn_gd_prefill(_padded(q[3][pl:], dk).to(DEV), _padded(k[3][pl:], dk).to(DEV), _padded(v[3][pl:], dv).to(DEV), [n - pl], L,
                            scale, work=_work([n - pl], DEV), window=window,
                            prefix=(_padded(k[3][:pl], dk).to(DEV), _padded(v[3][:pl], dv).to(DEV),
                                    torch.tensor([pl], dtype=torch.int32, device=DEV), [pl]))
    _close(o[:, :H * dv].view(-1, H, dv)[..., :D], full[3][pl:], tol)
    # decode: every sequence's last token
    P = 16
    pages = sum(-(-m // P) for m in lens)
    perm, at = torch.randperm(pages, generator=g), 0
    kc, vc = (torch.zeros(pages, G, P, d, dtype=dtype, device=DEV) for d in (dk, dv))
    bt = torch.zeros(4, 19, dtype=torch.int32)
    for i, m in enumerate(lens):
        own = perm[at:at + -(-m // P)]
        at += len(own)
        bt[i, :len(own)] = own.to(torch.int32)
        rows = torch.zeros(m, L.ncol)
        rows[:, H * dk:(H + G) * dk] = _padded(k[i].float(), dk).reshape(m, -1)
        rows[:, (H + G) * dk:(H + G) * dk + G * dv] = _padded(v[i].float(), dv).reshape(m, -1)
        slots = torch.tensor([int(own[j // P]) * P + j % P for j in range(m)])
        LN = dec.HeadLayout(H, G, D, D, 0, False)
        dec.qkv_heads(rows.to(dtype).to(DEV), torch.arange(m, device=DEV), None, LN, dtype, cache=(kc, vc), slots=slots.to(DEV))
    gd = torch.sigmoid(_rand(g, 4, H))
    want = torch.stack([f[-1] for f in full]) * gd.double()[..., None]
    for splits in (1, 2, 8):
        o = dec.attn_gd_decode(torch.stack([_padded(a[-1], dk) for a in q]).to(DEV), (kc, vc), bt.to(DEV),
                               torch.tensor(lens, dtype=torch.int32, device=DEV), L, scale, splits, window=window, gate=gd.to(DEV))
        _close(o[:, :H * dv].view(4, H, dv)[..., :D], want, tol)


# ---------------------------------------------------------------- latent attention
LATENT = [(4, 24, 8, 40, 72, 48), (1, 16, 2, 16, 33, 17), (16, 40, 12, 24, 128, 100), (17, 64, 64, 64, 200, 256), (40, 96, 32, 100, 64, 384),
          (32, 128, 64, 128, 256, 512), (6, 32, 96, 32, 64, 544)]


@pytest.mark.parametrize("H,D,R_,V,qr,kr", LATENT)
@pytest.mark.parametrize("own", [True, False])
@pytest.mark.parametrize("T", [3, 1100])
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_latent_rows_and_rotation(H, D, R_, V, qr, kr, own, T, dtype):
    if T > 100 and DEV == "cpu":
        pytest.skip("rows per workgroup are the GPU's")
    g = _g(H + kr)
    L = dec.LatentLayout(H, D, R_, V, qr, kr, own, 1e-5)
    n, P = L.ncol, 16
    real = torch.zeros(n)
    real[:qr] = 1
    at = L.qp
    if own:
        real[at:at + kr] = real[at + L.rp:at + L.rp + R_] = 1
        at += L.rp + L.rotp
    real[at:at + H] = 1
    x = (_rand(g, T, n) * real).to(dtype)
    qw, cw = torch.zeros(L.qp), torch.zeros(L.rp)
    qw[:qr], cw[:kr] = 1 + 0.2 * _rand(g, qr), 1 + 0.2 * _rand(g, kr)
    pos = torch.cat([torch.tensor([0, 999, 500]), torch.arange(T - 3) % 1000])
    tabs = dec.rotary_tables(1000, 20000.0, R_, device=DEV)
    pages = -(-T // P) + 1
    cache = torch.full((pages, 1, P, L.ck), 5.0, dtype=dtype, device=DEV)
    slots = torch.randperm(pages * P, generator=g)[:T]
    slots[1] = -1
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    z = x.double()
    for src in (x.to(DEV), ops.SplitK(torch.cat([x.float() * 0.5] * 2).reshape(-1).to(DEV), 2, T, n) if DEV == "cuda" else x):
        cq, gate, lat = dec.latent_rows(src, pos.to(DEV), tabs, L, dtype, qw.to(DEV), cw.to(DEV) if own else None, cache if own else None,
                                        slots.to(DEV))
        _close(cq[:, :qr], R.rms(z[:, :qr], 1e-5, qw[:qr].double()), tol)
        assert cq[:, qr:].abs().sum().item() == 0
        _close(gate, torch.sigmoid(z[:, at:at + H]), tol)
        if not own:
            assert lat is None
            continue
        _close(lat[:, :kr], R.rms(z[:, L.qp:L.qp + kr], 1e-5, cw[:kr].double()), tol)
        few = slice(0, 8)
        rot = R.rotate_half(z[few, None, L.qp + L.rp:L.qp + L.rp + R_], pos[few].tolist(), 20000.0)[:, 0]
        _close(lat[few, L.rp:L.rp + R_], rot, tol)
        assert lat[:, kr:L.rp].abs().sum().item() == 0 and lat[:, L.rp + R_:].abs().sum().item() == 0
        flat = cache.view(-1, L.ck)
        ok = slots >= 0
        assert torch.equal(flat[slots[ok].to(DEV)], lat[ok.to(DEV)])
        rest = torch.ones(pages * P, dtype=torch.bool)
        rest[slots[ok]] = False
        assert (flat.cpu()[rest] == 5.0).all()
    dk = L.pads[0]
    q = (_rand(g, T, H * dk)).to(dtype)
    qr_ = q.double().view(T, H, dk)
    want = torch.cat([qr_[:8, :, :D], R.rotate_half(qr_[:8, :, D:D + R_], pos[:8].tolist(), 20000.0), qr_[:8, :, D + R_:]], -1)
    got = dec.rotate_heads(q.clone().to(DEV), pos.to(DEV), tabs, L, dtype)
    _close(got[:8], want, tol)
    if DEV == "cuda":
        again = dec.rotate_heads(ops.SplitK(torch.cat([q.float() * 0.25, q.float() * 0.75]).reshape(-1).to(DEV), 2, T, H * dk), pos.to(DEV), tabs, L, dtype)
        _close(again, got, tol)


@pytest.mark.parametrize("H,D,R_,V,qr,kr", LATENT)
@pytest.mark.parametrize("page", [16, 64])
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_latent_decode(H, D, R_, V, qr, kr, page, dtype):
    """Decode attention in the latent space against keys and values expanded per head."""
    g = _g(H + kr + page)
    L = dec.LatentLayout(H, D, R_, V, qr, kr)
    dk, dv = L.pads
    lens = [1, 15, 16, 17, 63, 64, 65, 130, 0, 300]
    B, mp = len(lens), -(-304 // page)
    total = sum(-(-n // page) for n in lens)
    perm, at = torch.randperm(total + 2, generator=g), 0
    cache = torch.full((total + 2, 1, page, L.ck), float("inf") if dtype == torch.bfloat16 else 9.0, dtype=dtype, device=DEV)
    bt = torch.zeros(B, mp, dtype=torch.int32)
    uk, uv = _rand(g, H, D, kr, scale=kr ** -0.5).to(dtype), _rand(g, H, V, kr, scale=kr ** -0.5).to(dtype)
    q = torch.zeros(B, H, dk)
    q[..., :D + R_] = _rand(g, B, H, D + R_)
    q = q.to(dtype)
    scale, want = 2.0 / (D + R_) ** 0.5, []
    for b, n in enumerate(lens):
        own = perm[at:at + -(-n // page)]
        at += len(own)
        bt[b, :len(own)] = own.to(torch.int32)
        c, rot = _rand(g, n, kr).to(dtype), _rand(g, n, R_).to(dtype)
        row = torch.zeros(n, L.ck, dtype=dtype)
        row[:, :kr], row[:, L.rp:L.rp + R_] = c, rot
        for t in range(n):
            cache[int(own[t // page]), 0, t % page] = row[t].to(DEV)
        k = torch.cat([torch.einsum("tc,hdc->thd", c.double(), uk.double()), rot.double()[:, None].expand(n, H, R_)], -1)
        v = torch.einsum("tc,hdc->thd", c.double(), uv.double())
        s = torch.einsum("hd,thd->ht", q[b, :, :D + R_].double(), k) * scale
        want.append(torch.einsum("ht,thd->hd", torch.softmax(s, -1), v) if n else torch.zeros(H, V, dtype=torch.float64))
    gate = torch.sigmoid(_rand(g, B, H))
    want = torch.stack(want) * gate.double()[..., None]
    wabs = torch.zeros(H, L.rp, dec.pad_to(D, 16), dtype=dtype)
    wabs[:, :kr, :D] = uk.transpose(1, 2)
    wuv = torch.zeros(H, dv, L.rp, dtype=dtype)
    wuv[:, :V, :kr] = uv
    ql = dec.to_latent(q.to(DEV), wabs.to(DEV), L)
    _close(ql[..., :kr], torch.einsum("bhd,hdc->bhc", q[..., :D].double(), uk.double()), 2e-5 if dtype == torch.float32 else 1e-2)
    assert torch.equal(ql[..., L.rp:L.rp + R_].cpu(), q[..., D:D + R_]) and ql[..., L.rp + R_:].abs().sum().item() == 0
    for splits in (1, 2, 4):
        o = dec.attn_latent_decode(ql, cache, bt.to(DEV), torch.tensor(lens, dtype=torch.int32, device=DEV), L, scale, splits, gate=gate.to(DEV))
        y = dec.from_latent(o, wuv.to(DEV), L)
        got = y[:, :H * dv].view(B, H, dv)
        _close(got[..., :V], want, 5e-5 if dtype == torch.float32 else 2e-2)
        assert got[..., V:].abs().sum().item() == 0 and y[:, H * dv:].abs().sum().item() == 0
