"""Sufolix end to end against the plain implementation of its equations (sufolix_oracle):
configuration and loading, prefill, decoding through the paged cache, batches, page reuse,
scheduling and greedy generation. Every case runs on the CPU reference ops in fp32, and on the
GPU kernels in fp32 and bf16.
"""
import io
import json

import pytest
import torch
from safetensors.torch import save_file

import sufolix_oracle as O
from operator_amd.config import Settings
from operator_amd.engine.factory import build_engine
from operator_amd.engine.llm import GenRequest
from operator_amd.engine.replay import TraceReplay, replay
from operator_amd.models.config import config_from_dir, sufolix_from_dict
from operator_amd.models.kv_cache import PagedKVCache
from operator_amd.models.registry import build_model, model_class
from operator_amd.models.sufolix import SufolixModel

BACKENDS = [pytest.param(("cpu", "float32"), id="cpu"),
            pytest.param(("cuda", "float32"), id="gpu-fp32", marks=pytest.mark.gpu),
            pytest.param(("cuda", "bfloat16"), id="gpu-bf16", marks=pytest.mark.gpu)]


def attention(heads, kv, dim, vdim, rot, v_mix=True, sharp=8.0, base=1e4):
    """A mixer whose scores reach +-sharp: q and k are unit vectors times sqrt(dim)."""
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "rot": {"base": base, "dims": rot},
            "scale": sharp / dim, "v_mix": v_mix}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, n, top, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": n, "top": top}}
    return m if shared is None else {**m, "shared": {"ff": shared}}


def config(layers, width=160, vocab=300, streams=3, scale=5.0, eps=1e-5):
    return {"architecture": "Sufolix", "embedding": {"scale": scale}, "norm": {"eps": eps}, "streams": streams,
            "vocab": vocab, "width": width,
            "layers": [{"type": "attention", "mixer": a, "mlp": m} for a, m in layers]}


_A = attention(6, 2, 24, 40, 16)
CONFIGS = {
    # experts before dense, two of five experts, an expert layer first
    "mixed": config([(_A, moe(56, 5, 2, 72)), (_A, dense(200)), (_A, moe(40, 3, 3, 64)), (_A, dense(96))]),
    # every layer its own head layout; only some mix values, the first mixing layer is not the first layer
    "layouts": config([(attention(4, 4, 48, 16, 48, False), dense(128)), (attention(6, 3, 20, 24, 8, True, 12.0, 500.0), None),
                       (attention(3, 3, 32, 24, 32), moe(32, 4, 1)), (attention(5, 1, 80, 72, 2, False, 5.0), dense(72)),
                       (attention(9, 3, 16, 24, 16), moe(96, 2, 1, 40))], width=136, vocab=211, streams=2),
    # one stream, no mixing, a wide group
    "plain": config([(attention(20, 1, 32, 32, 32, False), dense(64)), (attention(2, 2, 64, 128, 20, False), moe(64, 7, 4, 128))],
                    width=64, vocab=128, streams=1, scale=1.0, eps=1e-6),
    "streams5": config([(_A, dense(64)), (_A, moe(64, 9, 1, 64))], width=192, streams=5),
}


def random_weights(cfg, seed=0):
    """bf16 tensors under the checkpoint's names: noticeable biases, gates, mixing and routing."""
    g = torch.Generator().manual_seed(seed)
    W, S, V = cfg["width"], cfg["streams"], cfg["vocab"]
    w = {}

    def add(name, *shape, std=None, mean=0.0):
        std = shape[-1] ** -0.5 if std is None else std
        w[name] = (mean + std * torch.randn(*shape, generator=g)).to(torch.bfloat16)

    def glu(p, ff):
        add(p + "gate", ff, W), add(p + "up", ff, W), add(p + "down", W, ff)

    add("embed", V, W, std=1.0)
    for i, lay in enumerate(cfg["layers"]):
        m, p = lay["mixer"], f"l{i}."
        for n, rows in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
            add(p + "mix." + n, rows, W)
            add(p + "mix." + n + ".b", rows, std=0.5)
        add(p + "mix.o", W, m["heads"] * m["vdim"])
        w[p + "mix.vmix"] = torch.tensor(0.2 + 0.15 * i).to(torch.bfloat16)
        for q in (1, 2) if lay["mlp"] else (1,):
            add(p + f"norm{q}", W, std=0.2, mean=1.0)
            add(p + f"hc{q}.in", S, std=0.3, mean=0.6)
            add(p + f"hc{q}.out", S, std=0.3, mean=0.8)
            w[p + f"hc{q}.mix"] = (torch.eye(S) + 0.25 * torch.randn(S, S, generator=g)).to(torch.bfloat16)
        f = lay["mlp"]
        if f and f["kind"] == "dense":
            glu(p + "mlp.", f["ff"])
        elif f:
            for e in range(f["router"]["experts"]):
                glu(p + f"mlp.e{e}.", f["expert"]["ff"])
            add(p + "mlp.router", f["router"]["experts"], W, std=3.0 * W ** -0.5)
            if f.get("shared"):
                glu(p + "mlp.shared.", f["shared"]["ff"])
                add(p + "mlp.shared.sg", 1, W, std=2.0 * W ** -0.5)
    add("final.norm", W, std=0.2, mean=1.0)
    add("head", V, W, std=2.0 * W ** -0.5)
    return w


def checkpoint(path, cfg, w):
    path.mkdir(exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(path / "model.safetensors"))
    return str(path)


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """name -> (config, weights, checkpoint directory, memo of oracle logits)."""
    root = tmp_path_factory.mktemp("sufolix")
    out = {}
    for i, (name, cfg) in enumerate(CONFIGS.items()):
        w = random_weights(cfg, i)
        out[name] = (cfg, w, checkpoint(root / name, cfg, w), {})
    return out


def oracle(m, tokens):
    """[T, vocab + 1]: the oracle's logits, and a last column that is 1 where every router chose
    with a clear gap (elsewhere rounding may send the token to another expert)."""
    cfg, w, _, memo = m
    key = tuple(tokens)
    if key not in memo:
        close: list = []
        lg = O.forward(cfg, w, list(tokens), close=close)
        gap = torch.stack(close).min(0)[0] if close else torch.ones(len(lg), dtype=lg.dtype)
        memo[key] = torch.cat([lg, (gap > 0.03).to(lg.dtype)[:, None]], 1)
    return memo[key]


def engine(m, backend, **kw):
    s = Settings()
    e = s.engine
    e.model, e.model_path, e.device, e.dtype = "t", m[2], *backend
    e.max_batch, e.max_context, e.max_prefill_tokens, e.kv_cache_gb = 8, 512, 512, 0.02
    pages = kw.pop("kv_pages", None)
    for k, v in kw.items():
        setattr(e, k, v)
    return build_engine(s, kv_pages=pages)[2]


def tokens(m, n, seed=0):
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, m[0]["vocab"], (n,), generator=g).tolist()


def check(got, want, backend):
    """Per row of ``oracle``'s: rms of the difference over the vocabulary, relative to the
    logits' spread (in bf16 where no router call was close)."""
    got, want, sure = got.double().cpu(), want[:, :-1].double(), want[:, -1] > 0
    assert got.shape == want.shape and torch.isfinite(got).all()
    d = got - want
    rel = ((d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.std(-1))
    if backend[1] == "bfloat16":
        rel = rel[sure]
        if not len(rel):
            return
    tol = {"float32": 2e-4, "bfloat16": 6e-2}[backend[1]]
    assert rel.max().item() < tol and (backend[1] == "float32" or rel.median().item() < 0.3 * tol), rel.tolist()


def run_given(eng, toks, cut):
    """Logits of every place: the first ``cut`` tokens as a prompt, the rest one by one."""
    (r,), lg = eng.given_start([toks[:cut]], [list(range(cut))])
    rows = [lg.float()] + [eng.given_next([r], [t]) for t in toks[cut:]]
    eng.given_end(r)
    return torch.cat(rows)


# ---------------------------------------------------------------- configuration and loading
def test_config_and_registry(models):
    for name, (cfg, w, path, _) in models.items():
        c = config_from_dir(path)
        assert c.arch == "sufolix" and model_class(c) is SufolixModel and c.layers == len(cfg["layers"])
        n = sum(t.numel() for k, t in w.items() if not k.endswith("vmix"))
        mixing = sum(1 for lay in cfg["layers"] if lay["mixer"]["v_mix"])
        assert c.param_count() == n + mixing
    bad = config([(attention(4, 3, 16, 16, 16), dense(64))])
    with pytest.raises(ValueError):
        sufolix_from_dict(bad)
    for key, value in (("type", "conv"), ("mlp", {"kind": "other"})):
        c = config([(_A, dense(64))])
        c["layers"][0][key] = value
        with pytest.raises(ValueError):
            sufolix_from_dict(c)
    with pytest.raises(ValueError):
        sufolix_from_dict(config([(_A, moe(32, 3, 4))]))
    with pytest.raises(ValueError):   # mixed values need one shape
        sufolix_from_dict(config([(attention(4, 2, 16, 16, 16), None), (attention(4, 2, 16, 24, 16), None)]))


def test_unknown_architecture(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Other"}))
    with pytest.raises(ValueError):
        config_from_dir(str(tmp_path))


def test_wrong_shape_is_refused(models, tmp_path):
    cfg, w, _, _ = models["streams5"]
    w = {**w, "l1.mix.k": w["l1.mix.k"][:, :-1].contiguous()}
    path = checkpoint(tmp_path / "bad", cfg, w)
    with pytest.raises(ValueError, match="l1.mix.k"):
        build_model(config_from_dir(path), device="cpu", dtype=torch.float32).load_checkpoint(path)


def test_weight_cache(models, tmp_path):
    from operator_amd.models import weight_cache

    path = models["layouts"][2]
    a, b = (build_model(config_from_dir(path), device="cpu", dtype=torch.float32) for _ in range(2))
    assert weight_cache.load_or_build(a, str(tmp_path), path, 0) == "miss"
    assert weight_cache.load_or_build(b, str(tmp_path), path, 0) == "hit"
    assert a.weight_bytes() == b.weight_bytes()
    for x, y in zip(a.layers, b.layers):
        for f in weight_cache.layer_fields(a):
            p, q = getattr(x, f), getattr(y, f)
            assert (p is None and q is None) or torch.equal(p, q), f


def test_cache_bytes(models):
    path = models["layouts"][2]
    m = build_model(config_from_dir(path), device="cpu", dtype=torch.float32)
    kv = PagedKVCache.for_model(m, 3, 16)
    assert [tuple(k.shape) for k in kv.k] == [(3, h, 16, d) for h, d, _ in m.kv_shapes()]
    assert [tuple(v.shape) for v in kv.v] == [(3, h, 16, d) for h, _, d in m.kv_shapes()]
    per = sum(h * (dk + dv) for h, dk, dv in m.kv_shapes()) * 16 * 4
    assert PagedKVCache.pages_for_shapes(10 * per + 1, m.kv_shapes(), 16, 4) == 10


# ---------------------------------------------------------------- logits
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_prompt_and_decode(models, backend, name):
    """A whole prompt, and prompts cut at page borders and elsewhere, then token by token."""
    m = models[name]
    eng = engine(m, backend)
    toks = tokens(m, 70)
    want = oracle(m, toks)
    for cut in (70, 64, 33, 16, 15, 1):
        check(run_given(eng, toks, cut), want, backend)
    assert eng.kv.allocator.free == eng.kv.num_pages


@pytest.mark.parametrize("backend", BACKENDS)
def test_residual_after_every_layer(models, backend):
    from operator_amd.models.base import ForwardBatch

    m = models["layouts"]
    eng = engine(m, backend)
    toks = tokens(m, 21)
    ref: list = []
    O.forward(m[0], m[1], toks, layer_out=ref)
    got: list = []
    r = GenRequest(toks)
    eng._reserve(r)
    p = eng._pack_prefill([r])
    t = eng._to_device
    work = (t(p["cu"], torch.int32), t(p["ws"], torch.int32), t(p["wq"], torch.int32), p["var"])
    fb = ForwardBatch(t(p["ids"]), t(p["pos"]), t(p["slots"]), True, t([20]), seq_lens=p["lens"],
                      prefill_work=work if backend[0] == "cuda" else None, residual_sink=lambda i, x: got.append(x))
    lg = eng.model.forward(fb, eng.kv)
    check(lg, oracle(m, toks)[20:], backend)
    sure = oracle(m, toks)[:, -1] > 0
    assert len(got) == len(ref)
    for a, b in zip(got, ref):
        rel = ((a.double().cpu() - b)[sure].pow(2).mean().sqrt() / b.pow(2).mean().sqrt()).item()
        assert rel < (1e-5 if backend[1] == "float32" else 2e-2)


@pytest.mark.parametrize("backend", BACKENDS)
def test_unequal_batch_matches_each_alone(models, backend):
    m = models["mixed"]
    eng = engine(m, backend)
    prompts = [tokens(m, n, n) for n in (1, 130, 16, 47, 2)]
    tails = [tokens(m, 20, 100 + n) for n in range(5)]
    want = [oracle(m, p + t) for p, t in zip(prompts, tails)]
    reqs, lg = eng.given_start(prompts, [list(range(len(p))) for p in prompts])
    check(lg, torch.cat([w[:len(p)] for w, p in zip(want, prompts)]), backend)
    live = list(range(5))
    for i in range(20):
        got = eng.given_next([reqs[j] for j in live], [tails[j][i] for j in live])
        check(got, torch.stack([want[j][len(prompts[j]) + i] for j in live]), backend)
        if i in (3, 8, 15):   # shorter requests end earlier; the others go on
            eng.given_end(reqs[live.pop(1)])
    for j in live:
        eng.given_end(reqs[j])
    assert eng.kv.allocator.free == eng.kv.num_pages


@pytest.mark.parametrize("backend", BACKENDS)
def test_pages_are_reused(models, backend):
    """A cache of few pages, handed from request to request with other lengths: nothing of an
    earlier owner shows."""
    m = models["layouts"]
    eng = engine(m, backend, kv_pages=6)
    for seed, (n, cut) in enumerate(((90, 80), (17, 3), (33, 16), (96, 96), (5, 1), (64, 31))):
        toks = tokens(m, n, 20 + seed)
        check(run_given(eng, toks, cut), oracle(m, toks), backend)
    with pytest.raises(MemoryError):
        eng.given_start([tokens(m, 200)], [[0]])


@pytest.mark.parametrize("backend", BACKENDS)
def test_long_decode_crosses_pages(models, backend):
    m = models["streams5"]
    eng = engine(m, backend)
    toks = tokens(m, 150, 5)
    check(run_given(eng, toks, 3), oracle(m, toks), backend)


def aim(cfg, w, pairs):
    """Make layer 0's keys such that token B's key is token A's query for every (A, B) of
    ``pairs``: with sharp scores, A reads B and little else, however far away B is."""
    m = cfg["layers"][0]["mixer"]
    per = m["heads"] // m["kv_heads"]
    w["l0.mix.q.b"], w["l0.mix.k.b"] = torch.zeros_like(w["l0.mix.q.b"]), torch.zeros_like(w["l0.mix.k.b"])

    def h(tok):   # the mixer's input in layer 0 depends on the token alone
        x = w["embed"][tok].double() * cfg["embedding"]["scale"] * w["l0.hc1.in"].double().sum()
        return O.rms(x, cfg["norm"]["eps"], w["l0.norm1"].double())

    q = w["l0.mix.q"].double().view(m["heads"], m["dim"], -1)[::per].reshape(-1, cfg["width"])
    A, B = (torch.stack([h(p[n]) for p in pairs]) for n in (0, 1))
    k = w["l0.mix.k"].double()
    w["l0.mix.k"] = (k + torch.linalg.lstsq(B, A @ q.T - B @ k.T).solution.T).to(torch.bfloat16)


@pytest.mark.parametrize("backend", BACKENDS)
def test_far_key_decides(models, backend, tmp_path):
    """Scores so sharp that one token takes most of the attention of one other, hundreds of
    places on: at the first tokens, on both sides of page and tile borders, right before the
    query; whether it is read shows far above rounding, in prompts and in decoding."""
    cfg = config([(attention(4, 2, 32, 32, 2, True, 60.0, 1e6), None), (attention(4, 2, 32, 32, 2), dense(64))], scale=0.2,
                 width=64, vocab=150, streams=2)
    w = random_weights(cfg, 3)
    place = {299: 0, 298: 1, 297: 15, 296: 16, 295: 31, 294: 32, 293: 63, 292: 64, 291: 127, 290: 128, 289: 255, 288: 256,
             287: 286, 70: 0}   # query position -> key position
    spots = sorted({*place.values()})
    key_tok = {p: i for i, p in enumerate(spots)}               # tokens 0.. stand at the key positions only
    query_tok = {q: 20 + i for i, q in enumerate(place)}
    aim(cfg, w, [(query_tok[q], key_tok[p]) for q, p in place.items() if q != 70])
    query_tok[70] = query_tok[299]
    m = (cfg, w, checkpoint(tmp_path / "far", cfg, w), {})
    g = torch.Generator().manual_seed(9)
    toks = torch.randint(50, 150, (300,), generator=g).tolist()
    for q, p in place.items():
        toks[q], toks[p] = query_tok[q], key_tok[p]
    want = oracle(m, toks)
    for q, p in place.items():
        other = list(toks)
        other[p] = 149   # without its token the query's logits are others
        assert (O.forward(cfg, w, other, dtype=torch.float32)[q] - want[q, :-1]).std() > 0.3 * want[q, :-1].std(), (q, p)
    eng = engine(m, backend)
    for cut in (300, 280, 65):
        got = run_given(eng, toks, cut)
        check(got[list(place)], want[list(place)], backend)


@pytest.mark.parametrize("backend", BACKENDS)
def test_given_steps_refuse_what_they_cannot_hold(models, backend):
    eng = engine(models["plain"], backend, max_context=32)
    with pytest.raises(ValueError, match="max_context"):
        eng.given_start([list(range(40))], [[0]])


# ---------------------------------------------------------------- generation
def check_greedy(m, prompt, output, backend):
    """Every generated token is the oracle's best continuation (a near tie may fall either way)."""
    lg = O.forward(m[0], m[1], list(prompt) + output[:-1], dtype=torch.float32)[len(prompt) - 1:]
    gap = (lg.max(1)[0] - lg.gather(1, torch.tensor(output)[:, None])[:, 0]) / lg.std(1)
    assert gap.max().item() < (1e-3 if backend[1] == "float32" else 0.15), gap.tolist()


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("sharing", [False, True])
def test_greedy_generation_through_the_scheduler(models, backend, sharing):
    """More requests than rows, unequal prompts, cancelled and late ones: each gets the tokens it
    would get alone (prompts share a head, so prefix sharing takes part when it is on)."""
    m = models["mixed"]
    eng = engine(m, backend, max_batch=4, prefix_sharing=sharing)
    head = tokens(m, 48, 77)
    prompts = [head + tokens(m, n, 40 + n) for n in (1, 9)] + [tokens(m, n, 60 + n) for n in (1, 17, 100)] \
        + [head + tokens(m, n, 40 + n) for n in (30, 5)]
    reqs = [eng.submit(GenRequest(p, max_tokens=8, temperature=0.0, ignore_eos=True)) for p in prompts[:2]]
    eng.step()
    reqs += [eng.submit(GenRequest(p, max_tokens=8, temperature=0.0, ignore_eos=True)) for p in prompts[2:]]
    gone = eng.submit(GenRequest(tokens(m, 20), max_tokens=8))
    eng.cancel(gone)
    for _ in range(200):
        if all(r.done for r in reqs):
            break
        eng.step()
    assert gone.error == "cancelled"
    for p, r in zip(prompts, reqs):
        assert r.error is None and len(r.output) == 8
        check_greedy(m, p, r.output, backend)
    held = eng.prefix_pages
    assert eng.kv.allocator.free + held == eng.kv.num_pages
    assert (eng.stats.prefix_hits > 0) == sharing


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_graph_replays_match_eager(models, dtype):
    """Captured graphs, replayed several times with eager work and synchronisation between:
    decode steps bit for bit as without a graph, whole generations the same every time."""
    m = models["mixed"]
    prompts = [tokens(m, n, n) for n in (40, 3, 77)]
    tails = [tokens(m, 10, 50 + n) for n in range(3)]

    def decode(use_graphs):
        eng = engine(m, ("cuda", dtype), use_graphs=use_graphs)
        out = []
        for _ in range(3):
            reqs, _ = eng.given_start(prompts, [[0]] * 3)
            for i in range(10):
                out.append(eng.given_next(reqs, [t[i] for t in tails]))
                torch.randn(1000, device="cuda").sum().item()
            for r in reqs:
                eng.given_end(r)
        return torch.stack(out)

    a, b = decode(True), decode(False)
    assert torch.equal(a, b) and torch.equal(a[:10], a[10:20]) and torch.equal(a[:10], a[20:])
    eng = engine(m, ("cuda", dtype), prefix_sharing=False)
    outs = []
    for _ in range(3):
        reqs = [GenRequest(p, max_tokens=12, temperature=0.8, seed=5, ignore_eos=True) for p in prompts]
        eng.generate(reqs)
        torch.randn(1000, device="cuda").sum().item()
        outs.append([r.output for r in reqs])
    assert eng.stats.graph_replays > 0 and eng.stats.prefill_graph_replays == 3
    assert outs[0] == outs[1] == outs[2]


# ---------------------------------------------------------------- trace replay
@pytest.mark.parametrize("backend", BACKENDS)
def test_replay_command(models, backend, tmp_path, capsys):
    m = models["layouts"]
    a, b = tokens(m, 30, 1), tokens(m, 12, 2)
    want = {"a": oracle(m, a), "b": oracle(m, b)}
    steps = [{"step": 0, "entries": [{"id": "b", "tokens": b[:10], "want": [9, 0]}, {"id": "a", "tokens": a[:20], "want": []}],
              "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [a[20]], "want": [0]}, {"id": "b", "tokens": [b[10]], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": [a[21]], "want": []}, {"id": "b", "tokens": [b[11]], "want": []}], "end": ["b"]}]
    steps += [{"step": 3 + i, "entries": [{"id": "a", "tokens": [t], "want": [0]}], "end": ["a"] if i == 7 else []}
              for i, t in enumerate(a[22:30])]
    steps.append({"step": 11, "entries": [{"id": "b", "tokens": b, "want": [11]}], "end": ["b"]})
    s = Settings()
    s.engine.device = backend[0]
    rc = replay(m[2], backend[1], str(tmp_path / "out"), 64, s, io.StringIO("\n".join(json.dumps(x) for x in steps) + "\n"))
    assert rc == 0
    assert [x for x in capsys.readouterr().out.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(12)]

    def rows(i):
        return torch.frombuffer(bytearray((tmp_path / "out" / f"{i}.f32").read_bytes()), dtype=torch.float32).view(-1, m[0]["vocab"])

    check(rows(0), want["b"][[9, 0]], backend)
    check(rows(1), torch.stack([want["a"][20], want["b"][10]]), backend)
    assert not (tmp_path / "out" / "2.f32").exists()
    for i in range(8):
        check(rows(3 + i), want["a"][22 + i:23 + i], backend)
    check(rows(11), want["b"][11:], backend)


def test_replay_refuses_a_mixed_step(models):
    rp = TraceReplay(engine(models["plain"], ("cpu", "float32")))
    rp.step([{"id": "a", "tokens": [1, 2], "want": []}], [])
    with pytest.raises(ValueError):
        rp.step([{"id": "a", "tokens": [1], "want": []}, {"id": "b", "tokens": [1], "want": []}], [])


def test_served_as_the_explanation_model(tmp_path):
    """The preset through the settings, the tokenizer and the explanation engine."""
    from operator_amd.engine.factory import build_llm

    s = Settings()
    e = s.engine
    e.model, e.device, e.dtype, e.max_batch, e.max_context, e.kv_cache_gb = "tiny-sufolix", "cpu", "float32", 2, 128, 0.01
    model, kv, llm, tok = build_llm(s)
    ids = tok.encode("OOMKilled: container exceeded its memory limit")
    r = llm.generate([GenRequest(ids, max_tokens=4, temperature=0.7, seed=3, ignore_eos=True)])[0]
    assert len(r.output) == 4 and all(0 <= t < model.cfg.vocab_size for t in r.output)
