"""Relurax end to end against the plain implementation of its equations (relurax_oracle):
configuration and loading, prefill, decoding through the paged cache and its page state, batches,
page reuse, window edges, shared latent rows, scheduling and greedy generation. Every case runs
on the CPU reference ops in fp32, and on the GPU kernels in fp32 and bf16.
"""
import io
import json

import pytest
import torch
from safetensors.torch import save_file

import relurax_oracle as O
from operator_amd.config import Settings
from operator_amd.engine.factory import build_engine
from operator_amd.engine.llm import GenRequest
from operator_amd.engine.replay import replay
from operator_amd.models.config import config_from_dir, get_config, relurax_from_dict
from operator_amd.models.kv_cache import PagedKVCache
from operator_amd.models.registry import build_model, model_class
from operator_amd.models.relurax import ReluraxModel

BACKENDS = [pytest.param(("cpu", "float32"), id="cpu"),
            pytest.param(("cuda", "float32"), id="gpu-fp32", marks=pytest.mark.gpu),
            pytest.param(("cuda", "bfloat16"), id="gpu-bf16", marks=pytest.mark.gpu)]


def attn(heads, kv, dim, window, taps=3, sharp=6.0):
    """A window layer whose scores reach about +-sharp (q and k are unit vectors times sqrt(dim))."""
    return "attention", {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "conv": taps, "mask": {"size": window},
                         "scale": sharp / dim}


def latent(heads, dim, rot, vdim, q_rank, kv_rank, base=1e4, scale=0.3, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
         "rot": {"base": base, "dims": rot}}
    return "latent_attention", m if kv_from is None else {**m, "kv_from": kv_from}


def config(layers, width=160, vocab=300, eps=1e-5):
    return {"architecture": "Relurax", "norm": {"eps": eps}, "vocab": vocab, "width": width,
            "layers": [{"type": t, "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}} for (t, m), ff in layers]}


CONFIGS = {
    # latent layers first, last and in between; the fourth layer reads the first one's rows
    "mixed": config([(latent(5, 24, 12, 40, 72, 56), 200), (attn(6, 2, 40, 24), 96), (attn(4, 4, 16, 70, 2), None),
                     (latent(3, 48, 12, 16, 100, 56, kv_from=0), 72), (attn(3, 1, 56, 33, 5), 150)]),
    # every window its own size, down to the token itself; one to eight taps
    "windows": config([(attn(4, 2, 24, 1, 4), 64), (attn(6, 3, 32, 16, 1), None), (attn(8, 1, 64, 17, 8), 128),
                       (attn(2, 2, 100, 64, 3), 72)], width=136, vocab=211, eps=1e-6),
    # several latent layers of different sizes, two chains of shared rows, one head, many heads
    "latents": config([(latent(1, 16, 2, 24, 40, 32), 64), (latent(20, 16, 32, 16, 200, 160, 500.0, 0.2), None),
                       (latent(4, 40, 2, 64, 64, 32, kv_from=0), 96), (latent(34, 24, 32, 8, 24, 160, 500.0, 0.25, kv_from=1), 64)],
                      width=192, vocab=128),
    # nothing but one window layer wider than any prompt
    "single": config([(attn(5, 5, 96, 1000, 3), 40)], width=64, vocab=97),
}


def random_weights(cfg, seed=0):
    """bf16 tensors under the checkpoint's names: noticeable taps, gates and norm weights."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    w = {}

    def add(name, *shape, std=None, mean=0.0):
        std = shape[-1] ** -0.5 if std is None else std
        w[name] = (mean + std * torch.randn(*shape, generator=g)).to(torch.bfloat16)

    add("embed", V, W, std=1.0)
    for i, lay in enumerate(cfg["layers"]):
        m, p = lay["mixer"], f"l{i}.mix."
        H = m["heads"]
        if lay["type"] == "attention":
            for n, heads in (("q", H), ("k", m["kv_heads"])):
                add(p + n, heads * m["dim"], W)
                add(p + n + ".conv", heads * m["dim"], m["conv"], std=0.6)
                add(p + n + ".norm", m["dim"], std=0.2, mean=1.0)
        else:
            D, R, C = m["dim"], m["rot_dim"], m["kv_rank"]
            add(p + "dq", m["q_rank"], W), add(p + "dq.norm", m["q_rank"], std=0.2, mean=1.0)
            add(p + "uq", H * (D + R), m["q_rank"])
            if "kv_from" not in m:
                add(p + "dkv", C + R, W, std=1.5 * W ** -0.5), add(p + "dkv.norm", C, std=0.2, mean=1.0)
            add(p + "uk", H * D, C), add(p + "uv", H * m["vdim"], C)
        add(p + "g", H, W, std=2.0 * W ** -0.5)
        add(p + "o", W, H * m["vdim"])
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if lay["mlp"] else ()):
            add(f"l{i}.{n}", W, std=0.2, mean=1.0)
        if lay["mlp"]:
            ff = lay["mlp"]["ff"]
            add(f"l{i}.mlp.gate", ff, W), add(f"l{i}.mlp.up", ff, W), add(f"l{i}.mlp.down", W, ff)
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
    root = tmp_path_factory.mktemp("relurax")
    out = {}
    for i, (name, cfg) in enumerate(CONFIGS.items()):
        w = random_weights(cfg, i)
        out[name] = (cfg, w, checkpoint(root / name, cfg, w), {})
    return out


def oracle(m, toks):
    cfg, w, _, memo = m
    key = tuple(toks)
    if key not in memo:
        memo[key] = O.forward(cfg, w, list(toks))
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
    """Per row: rms of the difference over the vocabulary, relative to the logits' spread."""
    got, want = got.double().cpu(), want.double()
    assert got.shape == want.shape and torch.isfinite(got).all()
    d = got - want
    rel = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.std(-1)
    tol = {"float32": 2e-5, "bfloat16": 5e-2}[backend[1]]
    assert rel.max().item() < tol and rel.median().item() < 0.5 * tol, rel.tolist()


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
        assert c.arch == "relurax" and model_class(c) is ReluraxModel and c.layers == len(cfg["layers"])
        assert c.param_count() == sum(t.numel() for t in w.values())
        kept = sum(m["kv_rank"] + m["rot_dim"] if "kv_rank" in m else 2 * m["kv_heads"] * m["dim"]
                   for m in (lay["mixer"] for lay in cfg["layers"]) if "kv_from" not in m)
        assert c.kv_bytes_per_token() == 2 * kept


@pytest.mark.parametrize("layers", [
    [(attn(4, 3, 16, 8), 64)],                                                            # heads over kv heads
    [(attn(4, 2, 300, 8), 64)],                                                           # head size
    [(attn(4, 2, 16, 0), 64)],                                                            # empty window
    [(attn(4, 2, 16, 8, 9), 64)],                                                         # taps
    [(("attention", {**attn(4, 2, 16, 8)[1], "vdim": 24}), 64)],                          # values are the keys
    [(("recurrent", attn(4, 2, 16, 8)[1]), 64)],
    [(latent(4, 16, 3, 16, 32, 32), 64)],                                                 # odd rotation
    [(("latent_attention", {**latent(4, 16, 4, 16, 32, 32)[1], "rot": {"base": 1e4, "dims": 2}}), 64)],
    [(latent(4, 16, 64, 16, 32, 608), 64)],                                               # latent row too long
    [(latent(4, 16, 4, 16, 32, 32, kv_from=0), 64)],                                      # reads itself
    [(attn(4, 2, 16, 8), 64), (latent(4, 16, 4, 16, 32, 32, kv_from=0), 64)],             # reads a layer without rows
    [(latent(4, 16, 4, 16, 32, 32), 64), (latent(4, 16, 4, 16, 32, 64, kv_from=0), 64)],  # rows of another size
    [(latent(4, 16, 4, 16, 32, 32), 64), (latent(4, 16, 4, 16, 32, 32, 99.0, kv_from=0), 64)],   # another rotation
    [(latent(4, 16, 4, 16, 32, 32), 64), (latent(4, 16, 4, 16, 32, 32, kv_from=0), 64), (latent(4, 16, 4, 16, 32, 32, kv_from=1), 64)],
    [],
])
def test_unsupported_layers_are_refused(layers):
    with pytest.raises(ValueError):
        relurax_from_dict(config(layers))


def test_unsupported_feed_forward_is_refused():
    c = config([(attn(4, 2, 16, 8), 64)])
    c["layers"][0]["mlp"]["kind"] = "other"
    with pytest.raises(ValueError):
        relurax_from_dict(c)


def test_wrong_shape_is_refused(models, tmp_path):
    cfg, w, _, _ = models["latents"]
    w = {**w, "l2.mix.uk": w["l2.mix.uk"][:, :-1].contiguous()}
    path = checkpoint(tmp_path / "bad", cfg, w)
    with pytest.raises(ValueError, match="l2.mix.uk"):
        build_model(config_from_dir(path), device="cpu", dtype=torch.float32).load_checkpoint(path)


def test_weight_cache(models, tmp_path):
    from operator_amd.models import weight_cache

    path = models["mixed"][2]
    a, b = (build_model(config_from_dir(path), device="cpu", dtype=torch.float32) for _ in range(2))
    assert weight_cache.load_or_build(a, str(tmp_path), path, 0) == "miss"
    assert weight_cache.load_or_build(b, str(tmp_path), path, 0) == "hit"
    assert a.weight_bytes() == b.weight_bytes()
    for x, y in zip(a.layers, b.layers):
        for f in weight_cache.layer_fields(a):
            p, q = getattr(x, f), getattr(y, f)
            assert (p is None and q is None) or torch.equal(p, q), f


def test_cache_shapes(models):
    """One row per token in a latent layer, none where another layer's are read, state rows per page."""
    m = build_model(config_from_dir(models["mixed"][2]), device="cpu", dtype=torch.float32)
    kv = PagedKVCache.for_model(m, 3, 16)
    assert [kv.k[i].numel() > 0 for i in range(5)] == [True, True, True, False, True]
    assert kv.k[0].shape == (3, 1, 16, 128) and kv.v[0].numel() == 0
    assert [None if s is None else tuple(s.shape) for s in kv.state] == [None, (3, 2, 8 * 48), (3, 1, 8 * 16), None, (3, 4, 4 * 64)]
    per = sum(t.numel() for t in (*kv.k, *kv.v, *filter(lambda s: s is not None, kv.state))) // 3 * 4
    assert PagedKVCache.pages_for_shapes(10 * per + 1, m.kv_shapes(), 16, 4, m.page_rows()) == 10
    from operator_amd.engine.speed import cut

    assert cut(get_config("tiny-relurax"), 2).layers == 2
    with pytest.raises(ValueError):
        PagedKVCache.for_model(m, 3, 2)   # pages shorter than the state


# ---------------------------------------------------------------- logits
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_prompt_and_decode(models, backend, name):
    """A whole prompt, and prompts cut at page borders and elsewhere, then token by token."""
    m = models[name]
    eng = engine(m, backend)
    toks = tokens(m, 90)
    want = oracle(m, toks)
    for cut in (90, 64, 33, 16, 15, 2, 1):
        check(run_given(eng, toks, cut), want, backend)
    assert eng.kv.allocator.free == eng.kv.num_pages


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["mixed", "latents"])
def test_residual_after_every_layer(models, backend, name):
    from operator_amd.models.base import ForwardBatch

    m = models[name]
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
    check(eng.model.forward(fb, eng.kv), oracle(m, toks)[20:], backend)
    assert len(got) == len(ref)
    for a, b in zip(got, ref):
        rel = ((a.double().cpu() - b).pow(2).mean().sqrt() / b.pow(2).mean().sqrt()).item()
        assert rel < (1e-5 if backend[1] == "float32" else 2e-2)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["mixed", "windows"])
def test_unequal_batch_matches_each_alone(models, backend, name):
    m = models[name]
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
@pytest.mark.parametrize("name", ["mixed", "windows"])
def test_pages_are_reused(models, backend, name):
    """A cache of few pages, handed from request to request with other lengths: no row and no state
    of an earlier owner shows, and junk in free pages does not either."""
    m = models[name]
    eng = engine(m, backend, kv_pages=6)
    for t in (*eng.kv.k, *eng.kv.v, *(s for s in eng.kv.state if s is not None)):
        t.fill_(3.0)
    for seed, (n, cut) in enumerate(((90, 80), (17, 3), (33, 16), (96, 96), (5, 1), (64, 31))):
        toks = tokens(m, n, 20 + seed)
        check(run_given(eng, toks, cut), oracle(m, toks), backend)
    with pytest.raises(MemoryError):
        eng.given_start([tokens(m, 200)], [[0]])


@pytest.mark.parametrize("backend", BACKENDS)
def test_long_decode_passes_windows_and_pages(models, backend):
    m = models["mixed"]
    eng = engine(m, backend)
    toks = tokens(m, 190, 5)
    check(run_given(eng, toks, 3), oracle(m, toks), backend)


def plain_taps(w, p):
    """Convolutions that pass the current token only."""
    for n in ("q", "k"):
        c = torch.zeros_like(w[p + n + ".conv"])
        c[:, -1] = 1
        w[p + n + ".conv"] = c


def first_input(cfg, w, tok):
    """The first layer's mixer input of a token: it depends on nothing else."""
    return O.rms(w["embed"][tok].double(), cfg["norm"]["eps"], w["l0.norm1"].double())


def planted(place, filler):
    """(tokens, query tokens, key tokens): distinct tokens at the query and key positions of ``place``."""
    keys = {p: i for i, p in enumerate(sorted({*place.values()}))}
    queries = {q: 30 + i for i, q in enumerate(place)}
    toks = list(filler)
    for q, p in place.items():
        toks[q], toks[p] = queries[q], keys[p]
    return toks, queries, keys


def far_effect(cfg, w, toks, q, p):
    """How much the logits at q change with the token at p, relative to their spread."""
    other = list(toks)
    other[p] = cfg["vocab"] - 1
    a, b = (O.forward(cfg, w, t, dtype=torch.float32)[q] for t in (toks, other))
    return ((a - b).std() / a.std()).item()


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("window", [33, 64, 97])
def test_window_edge_decides(backend, window, tmp_path):
    """One layer, scores so sharp that a key takes most of its query's attention: just inside the
    window it shows far above rounding, one place further nothing of it is left; in prompts and in
    decoding, over page and tile borders, also where the window starts with the sequence."""
    cfg = config([(attn(4, 2, 32, window, 4, 60.0), None)], width=64, vocab=150)
    w = random_weights(cfg, 3)
    plain_taps(w, "l0.mix.")
    w["l0.mix.g"] *= 0.1
    gone = {}
    place = {}
    for q in (window - 1, window, window + 15, 2 * window + 6, 199):   # query position -> key position
        place[q] = q - window + 1
    for q in (window + 2, window + 17, 2 * window + 9, 196):
        place[q] = q - window
        gone[q] = True
    used = set()
    place = {q: p for q, p in place.items() if p >= 0 and q < 200 and not ({q, p} & used or used.update((q, p)))}
    g = torch.Generator().manual_seed(9)
    toks, queries, keys = planted(place, torch.randint(60, 149, (200,), generator=g).tolist())
    m = cfg["layers"][0]["mixer"]
    q = w["l0.mix.q"].double().view(m["heads"], m["dim"], -1)[::2].reshape(-1, 64)
    A = torch.stack([first_input(cfg, w, queries[a]) for a in place])
    B = torch.stack([first_input(cfg, w, keys[b]) for b in place.values()])
    k = w["l0.mix.k"].double()
    w["l0.mix.k"] = (k + torch.linalg.lstsq(B, A @ q.T - B @ k.T).solution.T).to(torch.bfloat16)
    for a, b in place.items():
        e = far_effect(cfg, w, toks, a, b)
        assert e == 0 if a in gone else e > 0.2, (a, b, e)
    m = (cfg, w, checkpoint(tmp_path / "edge", cfg, w), {})
    want = oracle(m, toks)
    eng = engine(m, backend)
    for cut in (200, 190, window + 1, 20):
        got = run_given(eng, toks, cut)
        check(got[list(place)], want[list(place)], backend)


@pytest.mark.parametrize("backend", BACKENDS)
def test_far_latent_decides(backend, tmp_path):
    """Latent layers that share one layer's rows, scores sharp: single tokens hundreds of places back
    take most of a query's attention, at the first tokens, on both sides of page and tile borders and
    right before the query."""
    cfg = config([(latent(4, 32, 4, 32, 64, 96, scale=0.8), None), (latent(3, 24, 4, 40, 40, 96, kv_from=0), 64)], width=64, vocab=150)
    w = random_weights(cfg, 5)
    for n in ("uq",):   # the unrotated parts decide
        u = w["l0.mix." + n].view(4, 36, -1)
        u[:, 32:] *= 0.05
    w["l0.mix.g"] *= 0.1
    place = {299: 0, 298: 1, 297: 15, 296: 16, 295: 31, 294: 32, 293: 63, 292: 64, 291: 127, 290: 128, 289: 255, 288: 256, 287: 286}
    g = torch.Generator().manual_seed(9)
    toks, queries, keys = planted(place, torch.randint(60, 149, (300,), generator=g).tolist())
    wd = {k: v.double() for k, v in w.items()}
    eps, mx = cfg["norm"]["eps"], cfg["layers"][0]["mixer"]
    A = torch.stack([first_input(cfg, w, queries[a]) for a in place])
    B = torch.stack([first_input(cfg, w, keys[b]) for b in place.values()])
    q = (O.rms(A @ wd["l0.mix.dq"].T, eps, wd["l0.mix.dq.norm"]) @ wd["l0.mix.uq"].T).view(len(place), 4, 36)[..., :32].reshape(len(place), -1)
    c = O.rms(B @ wd["l0.mix.dkv"].T[:, :96], eps, wd["l0.mix.dkv.norm"])
    k = wd["l0.mix.uk"]
    w["l0.mix.uk"] = (k + torch.linalg.lstsq(c, q - c @ k.T).solution.T).to(torch.bfloat16)
    for a, b in place.items():
        assert far_effect(cfg, w, toks, a, b) > 0.2, (a, b)
    m = (cfg, w, checkpoint(tmp_path / "far", cfg, w), {})
    want = oracle(m, toks)
    eng = engine(m, backend)
    for cut in (300, 280, 65):
        got = run_given(eng, toks, cut)
        check(got[list(place)], want[list(place)], backend)


@pytest.mark.parametrize("backend", BACKENDS)
def test_given_steps_refuse_what_they_cannot_hold(models, backend):
    eng = engine(models["single"], backend, max_context=32)
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
@pytest.mark.parametrize("name", ["mixed", "windows"])
def test_greedy_generation_through_the_scheduler(models, backend, name, sharing):
    """More requests than rows, unequal prompts, cancelled and late ones: each gets the tokens it
    would get alone. Prompts share a head, so with prefix sharing their convolutions continue from
    the shared pages' state and their windows reach into the shared keys."""
    m = models[name]
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
    assert eng.kv.allocator.free + eng.prefix_pages == eng.kv.num_pages
    assert (eng.stats.prefix_hits > 0) == sharing


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["mixed", "windows"])
def test_prefill_after_a_shared_prefix(models, backend, name):
    """Logits of prompts computed behind a cached prefix, next to one computed whole."""
    m = models[name]
    eng = engine(m, backend, prefix_sharing=True)
    head = tokens(m, 32, 3)
    for _ in range(3):   # seen often enough, the head becomes a shared prefix
        eng.generate([GenRequest(head + [1, 2], max_tokens=1, temperature=0.0, ignore_eos=True)])
    assert eng.prefix_pages == 2
    prompts = [head + tokens(m, n, 30 + n) for n in (1, 2, 3, 40)] + [tokens(m, 19, 8)]
    reqs = [GenRequest(list(p), max_tokens=0) for p in prompts]
    for r in reqs[:4]:
        r.prefix = eng._pfx
        r.pages = list(eng._pfx.pages)
        eng._pfx.users += 1
    for r in reqs:
        eng._reserve(r)
    p = eng._pack_prefill(reqs)
    lg = eng._eager_prefill(p, list(range(len(p["ids"]))))
    want = torch.cat([oracle(m, t)[32:] for t in prompts[:4]] + [oracle(m, prompts[4])])
    check(lg, want, backend)
    tails = [tokens(m, 6, 80 + i) for i in range(5)]
    for i in range(6):
        got = eng.given_next(reqs, [t[i] for t in tails])
        check(got, torch.stack([oracle(m, a + b[:i + 1])[-1] for a, b in zip(prompts, tails)]), backend)
    for r in reqs:
        eng.given_end(r)


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
    for sharing in (False, True):
        eng = engine(m, ("cuda", dtype), prefix_sharing=sharing)
        outs = []
        for _ in range(3):
            reqs = [GenRequest(p, max_tokens=12, temperature=0.8, seed=5, ignore_eos=True) for p in prompts]
            eng.generate(reqs)
            torch.randn(1000, device="cuda").sum().item()
            outs.append([r.output for r in reqs])
        assert eng.stats.graph_replays > 0 and eng.stats.prefill_graph_replays >= 3
        if not sharing:
            assert outs[0] == outs[1] == outs[2]


@pytest.mark.gpu
def test_many_rows_and_splits():
    """Batches beyond one row tile and contexts cut into several pieces (prefill and decode of the preset)."""
    from operator_amd.engine.llm import LLMEngine

    m = build_model(get_config("tiny-relurax"), device="cuda").init_random(seed=2)
    prompts = [torch.randint(0, 900, (n,), generator=torch.Generator().manual_seed(n)).tolist() for n in range(700, 780)]

    def run(batch):
        eng = LLMEngine(m, PagedKVCache.for_model(m, 80 * 52, 16), max_batch=batch, max_prefill_tokens=8192, max_context=1024,
                        prefix_sharing=False)
        out = []
        for a in range(0, 80, batch):
            part = prompts[a:a + batch]
            reqs, lg = eng.given_start(part, [[len(p) - 1] for p in part])
            steps = [lg.float()] + [eng.given_next(reqs, [3 + i] * len(part)) for i in range(2)]
            for r in reqs:
                eng.given_end(r)
            out.append(torch.stack(steps, 1))
        return torch.cat(out).double()

    a, b = run(80), run(1)   # one split of the batch against many splits of a row
    d = a - b
    assert ((d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / b.std(-1)).max().item() < 4e-2


# ---------------------------------------------------------------- trace replay
@pytest.mark.parametrize("backend", BACKENDS)
def test_replay_command(models, backend, tmp_path, capsys):
    m = models["latents"]
    a, b = tokens(m, 30, 1), tokens(m, 12, 2)
    want = {"a": oracle(m, a), "b": oracle(m, b)}
    steps = [{"step": 0, "entries": [{"id": "b", "tokens": b[:10], "want": [9, 0]}, {"id": "a", "tokens": a[:20], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [a[20]], "want": [0]}, {"id": "b", "tokens": [b[10]], "want": [0]}],
              "end": ["b"]}]
    steps += [{"step": 2 + i, "entries": [{"id": "a", "tokens": [t], "want": [0]}], "end": ["a"] if i == 8 else []}
              for i, t in enumerate(a[21:30])]
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
    for i in range(9):
        check(rows(2 + i), want["a"][21 + i:22 + i], backend)
    check(rows(11), want["b"][11:], backend)


def test_served_as_the_explanation_model():
    """The preset through the settings, the tokenizer and the explanation engine."""
    from operator_amd.engine.factory import build_llm

    s = Settings()
    e = s.engine
    e.model, e.device, e.dtype, e.max_batch, e.max_context, e.kv_cache_gb = "tiny-relurax", "cpu", "float32", 2, 128, 0.01
    model, kv, llm, tok = build_llm(s)
    ids = tok.encode("OOMKilled: container exceeded its memory limit")
    r = llm.generate([GenRequest(ids, max_tokens=4, temperature=0.7, seed=3, ignore_eos=True)])[0]
    assert len(r.output) == 4 and all(0 <= t < model.cfg.vocab_size for t in r.output)
