"""Explanation-model configurations (Llama-architecture families, head_dim 128).

The reference delegates explanation to an external LLM via its ai-interface
service (J/service/AIInterfaceClient.java:45-59; AIProvider.spec.modelId), so
whichever model a user had behind that hop must be servable on-node. Supported
architectures share one decoder (pre-norm RMSNorm, RoPE, GQA, SwiGLU):

  llama    Llama-2/3/3.1/3.2 (llama3 rope scaling, tied embeddings for 3.2)
  mistral  Mistral-7B v0.2/v0.3 (no sliding window in those releases)
  qwen2    Qwen2 / Qwen2.5 (bias on the q/k/v projections, rms eps 1e-6)

BASELINE.json names Llama-3-8B (TP=1) and Llama-3-70B (TP=8) as the configs.
There are no checkpoints offline, so weights are random-initialised with the
exact architecture, or loaded from a local HF safetensors directory whose
``config.json`` then defines the architecture (``config_from_hf``).

  sufolix  Sufolix (``config_from_dir``): hyper-connected residual streams, attention layers
           with their own head sizes, per-head q/k norm and value mixing, dense or
           routed-expert feed-forwards; ``SufolixConfig``
  relurax  Relurax (``config_from_dir``): sliding-window attention whose values are its convolved
           keys, latent attention that may read another layer's cached rows, norms before and
           after every sublayer; ``ReluraxConfig``
"""
from __future__ import annotations

import json
import os
from dataclasses import asdict, dataclass, field, replace

ARCHS = ("llama", "mistral", "qwen2")


@dataclass(frozen=True)
class LlamaConfig:
    name: str = "llama3-8b"
    vocab_size: int = 128256
    hidden: int = 4096
    intermediate: int = 14336
    layers: int = 32
    heads: int = 32
    kv_heads: int = 8
    head_dim: int = 128
    rope_theta: float = 500000.0
    rms_eps: float = 1e-5
    max_position: int = 8192
    tie_embeddings: bool = False
    rope_scaling: dict | None = field(default=None, hash=False, compare=False)
    bos_id: int = 128000
    eos_ids: tuple[int, ...] = (128001, 128009)
    arch: str = "llama"
    qkv_bias: bool = False      # qwen2: q/k/v projections carry a bias
    add_bos: bool = True        # prepend bos_id to prompts (qwen2 tokenizers do not)

    @property
    def qkv_width(self) -> int:
        return (self.heads + 2 * self.kv_heads) * self.head_dim

    def param_count(self) -> int:
        h, i, v = self.hidden, self.intermediate, self.vocab_size
        per = h * self.qkv_width + self.heads * self.head_dim * h + 2 * h * i + i * h + 2 * h
        per += self.qkv_width if self.qkv_bias else 0
        return self.layers * per + v * h * (1 if self.tie_embeddings else 2) + h

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return self.layers * 2 * self.kv_heads * self.head_dim * dtype_bytes

    def to_dict(self) -> dict:
        return asdict(self)


_LLAMA31_SCALING = {"rope_type": "llama3", "factor": 8.0, "low_freq_factor": 1.0, "high_freq_factor": 4.0,
                    "original_max_position_embeddings": 8192}

PRESETS: dict[str, LlamaConfig] = {
    "llama3-8b": LlamaConfig(),
    "llama3.1-8b": LlamaConfig(name="llama3.1-8b", max_position=131072, rope_scaling=_LLAMA31_SCALING),
    "llama3-70b": LlamaConfig(name="llama3-70b", hidden=8192, intermediate=28672, layers=80, heads=64, kv_heads=8),
    "llama3.1-70b": LlamaConfig(name="llama3.1-70b", hidden=8192, intermediate=28672, layers=80, heads=64,
                                kv_heads=8, max_position=131072, rope_scaling=_LLAMA31_SCALING),
    "llama3.2-3b": LlamaConfig(name="llama3.2-3b", hidden=3072, intermediate=8192, layers=28, heads=24, kv_heads=8,
                               max_position=131072, tie_embeddings=True,
                               rope_scaling={**_LLAMA31_SCALING, "factor": 32.0}),
    "mistral-7b": LlamaConfig(name="mistral-7b", arch="mistral", vocab_size=32768, hidden=4096, intermediate=14336,
                              layers=32, heads=32, kv_heads=8, rope_theta=1e6, max_position=32768, bos_id=1,
                              eos_ids=(2,)),
    "qwen2.5-7b": LlamaConfig(name="qwen2.5-7b", arch="qwen2", vocab_size=152064, hidden=3584, intermediate=18944,
                              layers=28, heads=28, kv_heads=4, rope_theta=1e6, rms_eps=1e-6, max_position=32768,
                              qkv_bias=True, add_bos=False, bos_id=151643, eos_ids=(151645, 151643)),
    "qwen2.5-3b": LlamaConfig(name="qwen2.5-3b", arch="qwen2", vocab_size=151936, hidden=2048, intermediate=11008,
                              layers=36, heads=16, kv_heads=2, rope_theta=1e6, rms_eps=1e-6, max_position=32768,
                              tie_embeddings=True, qkv_bias=True, add_bos=False, bos_id=151643,
                              eos_ids=(151645, 151643)),
    # small configs with the same kernels (head_dim 128, GQA) for tests / quick runs
    "llama-1b-hd128": LlamaConfig(name="llama-1b-hd128", hidden=2048, intermediate=8192, layers=16, heads=16,
                                  kv_heads=4),
    "tiny": LlamaConfig(name="tiny", vocab_size=1024, hidden=256, intermediate=512, layers=2, heads=2, kv_heads=1,
                        max_position=4096, bos_id=1000, eos_ids=(1001,)),
    "tiny-gqa4": LlamaConfig(name="tiny-gqa4", vocab_size=2048, hidden=1024, intermediate=1024, layers=2, heads=8,
                             kv_heads=2, max_position=4096, bos_id=2000, eos_ids=(2001,)),
    # 70B-shaped head layout (GQA 8: 64/8 heads at 70B) that every TP degree up to 8 divides:
    # heads, kv heads, FFN width (64-feature SwiGLU blocks per rank) and vocab
    "tiny-tp8": LlamaConfig(name="tiny-tp8", vocab_size=2048, hidden=512, intermediate=1024, layers=2, heads=16,
                            kv_heads=8, max_position=4096, bos_id=2000, eos_ids=(2001,)),
    # qwen2-shaped: q/k/v bias and a GQA group of 7 (Qwen2.5-7B's 28/4)
    "tiny-qwen": LlamaConfig(name="tiny-qwen", arch="qwen2", vocab_size=2048, hidden=896, intermediate=1024, layers=2,
                             heads=7, kv_heads=1, rope_theta=1e6, rms_eps=1e-6, max_position=4096, qkv_bias=True,
                             add_bos=False, bos_id=2000, eos_ids=(2001,)),
}


@dataclass(frozen=True)
class AttentionSpec:
    """One attention mixer: head counts and sizes, rotary positions on the first ``rot_dims``
    dimensions, the score scale, and whether its values mix with the first mixing layer's.
    ``conv``: taps of a short causal convolution on q and k (0: none), ``window``: how far back a
    query sees, itself included (0: everything)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_base: float = 10000.0
    rot_dims: int = 0
    v_mix: bool = False
    conv: int = 0
    window: int = 0


@dataclass(frozen=True)
class LatentSpec:
    """One latent-attention mixer: queries from a latent of ``q_rank``, keys and values from one of
    ``kv_rank``; per head ``dim`` unrotated and ``rot_dim`` rotated query / key dimensions (all of the
    latter rotate) and ``vdim`` value ones. ``kv_from``: the layer whose cached rows it reads (-1: its own)."""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float = 10000.0
    kv_from: int = -1


@dataclass(frozen=True)
class FeedForwardSpec:
    """A SwiGLU feed-forward of ``ff`` features (experts == 0), or ``experts`` of them of which a
    token uses ``top``, with a shared one of ``shared_ff`` features (0: none)."""
    ff: int
    experts: int = 0
    top: int = 0
    shared_ff: int = 0


@dataclass(frozen=True)
class DecoderLayerSpec:
    mixer: AttentionSpec | LatentSpec
    mlp: FeedForwardSpec | None = None


@dataclass(frozen=True)
class SufolixConfig:
    name: str = "sufolix"
    vocab_size: int = 32000
    hidden: int = 1024
    streams: int = 4                 # parallel residual streams
    embed_scale: float = 1.0
    rms_eps: float = 1e-6
    layer_specs: tuple[DecoderLayerSpec, ...] = ()
    max_position: int = 32768        # rotary table length, not a limit of the design
    bos_id: int = -1
    eos_ids: tuple[int, ...] = (-1,)
    arch: str = "sufolix"
    add_bos: bool = False

    @property
    def layers(self) -> int:
        return len(self.layer_specs)

    def param_count(self) -> int:
        h, s = self.hidden, self.streams
        n = 2 * self.vocab_size * h + h
        for sp in self.layer_specs:
            a, m = sp.mixer, sp.mlp
            qkv = (a.heads + a.kv_heads) * a.dim + a.kv_heads * a.vdim
            n += qkv * (h + 1) + h * a.heads * a.vdim + h + s * (s + 2) + (1 if a.v_mix else 0)
            if m is not None:
                n += 3 * h * m.ff * max(1, m.experts) + h + s * (s + 2)
                n += h * m.experts + (3 * h * m.shared_ff + h if m.shared_ff else 0)
        return n

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return sum(sp.mixer.kv_heads * (sp.mixer.dim + sp.mixer.vdim) for sp in self.layer_specs) * dtype_bytes

    def to_dict(self) -> dict:
        return asdict(self)


@dataclass(frozen=True)
class ReluraxConfig:
    name: str = "relurax"
    vocab_size: int = 32000
    hidden: int = 1024
    rms_eps: float = 1e-6
    layer_specs: tuple[DecoderLayerSpec, ...] = ()
    max_position: int = 32768        # rotary table length, not a limit of the design
    bos_id: int = -1
    eos_ids: tuple[int, ...] = (-1,)
    arch: str = "relurax"
    add_bos: bool = False

    @property
    def layers(self) -> int:
        return len(self.layer_specs)

    def param_count(self) -> int:
        h = self.hidden
        n = 2 * self.vocab_size * h + h
        for sp in self.layer_specs:
            m = sp.mixer
            n += 2 * h + m.heads * h + m.heads * m.vdim * h
            if isinstance(m, LatentSpec):
                n += m.q_rank * (h + 1) + m.heads * (m.dim + m.rot_dim) * m.q_rank + m.heads * (m.dim + m.vdim) * m.kv_rank
                n += (m.kv_rank + m.rot_dim) * h + m.kv_rank if m.kv_from < 0 else 0
            else:
                n += (m.heads + m.kv_heads) * m.dim * (h + m.conv) + 2 * m.dim
            n += 3 * h * sp.mlp.ff + 2 * h if sp.mlp is not None else 0
        return n

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        n = 0
        for m in (sp.mixer for sp in self.layer_specs):
            if isinstance(m, LatentSpec):
                n += m.kv_rank + m.rot_dim if m.kv_from < 0 else 0
            else:
                n += m.kv_heads * (m.dim + m.vdim)
        return n * dtype_bytes

    def to_dict(self) -> dict:
        return asdict(self)


def _relurax(name: str, layers: int, attn: AttentionSpec, latent: LatentSpec, ff: int, **kw) -> ReluraxConfig:
    """Alternating window / latent layers; every second latent layer reads the one before it."""
    mix = [attn if i % 2 == 0 else latent if i % 4 == 1 else replace(latent, kv_from=i - 2) for i in range(layers)]
    return ReluraxConfig(name=name, layer_specs=tuple(DecoderLayerSpec(m, FeedForwardSpec(ff)) for m in mix), **kw)


def _sufolix(name: str, layers: int, mixer: AttentionSpec, dense: FeedForwardSpec, moe: FeedForwardSpec, **kw) -> SufolixConfig:
    """Alternating dense / expert layers of one mixer."""
    return SufolixConfig(name=name, layer_specs=tuple(DecoderLayerSpec(mixer, moe if i % 2 else dense)
                                                      for i in range(layers)), **kw)


DESIGN_PRESETS: dict[str, SufolixConfig | ReluraxConfig] = {
    "tiny-sufolix": _sufolix("tiny-sufolix", 4, AttentionSpec(6, 3, 40, 24, 0.2, 20000.0, 32, True),
                             FeedForwardSpec(160), FeedForwardSpec(72, experts=5, top=2, shared_ff=96),
                             vocab_size=1000, hidden=192, streams=3, embed_scale=8.0, bos_id=990, eos_ids=(991,)),
    # Llama-3-8B's widths and heads: the same projections per layer, hyper-connected, every
    # second feed-forward 8 experts of which 2 run (the active width stays near the dense one)
    "sufolix-8b": _sufolix("sufolix-8b", 32, AttentionSpec(32, 8, 128, 128, 0.088388, 500000.0, 128, True),
                           FeedForwardSpec(14336), FeedForwardSpec(4096, experts=8, top=2, shared_ff=4096),
                           vocab_size=128256, hidden=4096, streams=4, bos_id=128000, eos_ids=(128001, 128009)),
    # the width of a ~1B model with narrower values and a partial rotation
    "sufolix-1b": _sufolix("sufolix-1b", 16, AttentionSpec(16, 4, 128, 96, 0.1, 100000.0, 64, True),
                           FeedForwardSpec(8192), FeedForwardSpec(1024, experts=32, top=4, shared_ff=2048),
                           vocab_size=32000, hidden=2048, streams=4, bos_id=1, eos_ids=(2,)),
    "tiny-relurax": _relurax("tiny-relurax", 4, AttentionSpec(6, 2, 40, 40, 0.2, conv=4, window=24),
                             LatentSpec(5, 24, 8, 40, 72, 48, 0.25, 20000.0), 160,
                             vocab_size=1000, hidden=192, bos_id=990, eos_ids=(991,)),
    # Llama-3-8B's width, heads and feed-forward; latents of the usual large-model sizes
    "relurax-8b": _relurax("relurax-8b", 32, AttentionSpec(32, 8, 128, 128, 0.088388, conv=4, window=1024),
                           LatentSpec(32, 128, 64, 128, 1536, 512, 0.072169, 500000.0), 14336,
                           vocab_size=128256, hidden=4096, bos_id=128000, eos_ids=(128001, 128009)),
    # the width of a ~1B model, fewer and smaller heads
    "relurax-1b": _relurax("relurax-1b", 16, AttentionSpec(16, 4, 128, 128, 0.088388, conv=4, window=512),
                           LatentSpec(16, 96, 32, 96, 768, 256, 0.088388, 100000.0), 8192,
                           vocab_size=32000, hidden=2048, bos_id=1, eos_ids=(2,)),
}


def get_config(name: str, **overrides) -> "LlamaConfig | SufolixConfig | ReluraxConfig":
    if name in DESIGN_PRESETS:
        c = DESIGN_PRESETS[name]
    elif name in PRESETS:
        c = PRESETS[name]
    else:
        raise KeyError(f"unknown model preset {name!r}; known: {sorted([*PRESETS, *DESIGN_PRESETS])}")
    return replace(c, **overrides) if overrides else c


def _ids(v) -> tuple[int, ...]:
    if v is None:
        return ()
    return tuple(int(x) for x in (v if isinstance(v, (list, tuple)) else [v]))


def config_from_hf(path: str, name: str | None = None) -> LlamaConfig:
    """LlamaConfig from a HuggingFace checkpoint directory's ``config.json`` (plus the
    eos ids of ``generation_config.json`` when present). Raises ValueError for an
    architecture or shape the gfx950 kernels do not serve."""
    with open(os.path.join(path, "config.json")) as f:
        hc = json.load(f)
    mt = hc.get("model_type", "llama")
    if mt not in ARCHS:
        raise ValueError(f"{path}: model_type {mt!r} not supported (supported: {', '.join(ARCHS)})")
    heads = int(hc["num_attention_heads"])
    hidden = int(hc["hidden_size"])
    head_dim = int(hc.get("head_dim") or hidden // heads)
    if head_dim != 128:
        raise ValueError(f"{path}: head_dim {head_dim}; the attention kernels are built for head_dim 128")
    kv_heads = int(hc.get("num_key_value_heads") or heads)
    if heads % kv_heads or heads // kv_heads > 8:
        raise ValueError(f"{path}: GQA group {heads}/{kv_heads} not supported (1..8 query heads per kv head)")
    max_pos = int(hc.get("max_position_embeddings", 8192))
    sw = hc.get("sliding_window")
    if sw and (mt != "qwen2" or hc.get("use_sliding_window")):
        # full attention equals sliding-window attention while contexts stay inside the window
        max_pos = min(max_pos, int(sw))
    eos = _ids(hc.get("eos_token_id"))
    gen = os.path.join(path, "generation_config.json")
    if os.path.exists(gen):
        with open(gen) as f:
            eos = tuple(dict.fromkeys(eos + _ids(json.load(f).get("eos_token_id"))))
    rs = hc.get("rope_scaling")
    if rs is not None:
        rs = dict(rs)
        rs.setdefault("rope_type", rs.get("type"))
        if rs["rope_type"] not in ("llama3", "default", None):
            raise ValueError(f"{path}: rope_scaling type {rs['rope_type']!r} not supported")
        if rs["rope_type"] != "llama3":
            rs = None
    bos = hc.get("bos_token_id")
    return LlamaConfig(
        name=name or os.path.basename(os.path.normpath(path)), arch=mt, vocab_size=int(hc["vocab_size"]),
        hidden=hidden, intermediate=int(hc["intermediate_size"]), layers=int(hc["num_hidden_layers"]), heads=heads,
        kv_heads=kv_heads, head_dim=head_dim, rope_theta=float(hc.get("rope_theta", 10000.0)),
        rms_eps=float(hc.get("rms_norm_eps", 1e-5)), max_position=max_pos,
        tie_embeddings=bool(hc.get("tie_word_embeddings", False)), rope_scaling=rs,
        bos_id=int(bos) if bos is not None else -1, eos_ids=eos or (-1,),
        qkv_bias=bool(hc.get("attention_bias", mt == "qwen2")),
        add_bos=mt != "qwen2" and bos is not None)


def sufolix_from_dict(hc: dict, name: str = "sufolix") -> SufolixConfig:
    """SufolixConfig from a checkpoint's config.json contents."""
    specs = []
    for i, lay in enumerate(hc["layers"]):
        if lay["type"] != "attention":
            raise ValueError(f"layer {i}: mixer type {lay['type']!r} not supported")
        m, f = lay["mixer"], lay.get("mlp")
        rot = m.get("rot") or {"base": 1.0, "dims": 0}
        mixer = AttentionSpec(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                              scale=float(m["scale"]), rot_base=float(rot["base"]), rot_dims=int(rot["dims"]),
                              v_mix=bool(m.get("v_mix", False)))
        if mixer.heads % mixer.kv_heads:
            raise ValueError(f"layer {i}: {mixer.heads} query heads over {mixer.kv_heads} kv heads")
        if max(mixer.dim, mixer.vdim) > 256:
            raise ValueError(f"layer {i}: head sizes {mixer.dim}/{mixer.vdim}; the attention kernels go up to 256")
        if mixer.rot_dims % 2 or mixer.rot_dims > mixer.dim:
            raise ValueError(f"layer {i}: {mixer.rot_dims} rotated dimensions of {mixer.dim}")
        mlp = None
        if f is not None:
            if f["kind"] == "dense":
                mlp = FeedForwardSpec(int(f["ff"]))
            elif f["kind"] == "moe":
                mlp = FeedForwardSpec(int(f["expert"]["ff"]), experts=int(f["router"]["experts"]),
                                      top=int(f["router"]["top"]), shared_ff=int((f.get("shared") or {}).get("ff", 0)))
                if not 1 <= mlp.top <= mlp.experts <= 496:
                    raise ValueError(f"layer {i}: top {mlp.top} of {mlp.experts} experts")
            else:
                raise ValueError(f"layer {i}: feed-forward kind {f['kind']!r} not supported")
        specs.append(DecoderLayerSpec(mixer, mlp))
    shapes = {(sp.mixer.kv_heads, sp.mixer.vdim) for sp in specs if sp.mixer.v_mix}
    if len(shapes) > 1:
        raise ValueError(f"value-mixing layers disagree on the value shape: {sorted(shapes)}")
    streams = int(hc.get("streams", 1))
    if not specs or not 1 <= streams <= 8:
        raise ValueError(f"{len(specs)} layers, {streams} residual streams (1..8 supported)")
    return SufolixConfig(name=name, vocab_size=int(hc["vocab"]), hidden=int(hc["width"]), streams=streams,
                         embed_scale=float((hc.get("embedding") or {}).get("scale", 1.0)),
                         rms_eps=float(hc["norm"]["eps"]), layer_specs=tuple(specs))


def _heads(i: int, m: dict, dim: int) -> None:
    if int(m["heads"]) < 1 or max(dim, int(m["vdim"])) > 256:
        raise ValueError(f"layer {i}: head sizes {dim}/{m['vdim']}; the attention kernels go up to 256")


def relurax_from_dict(hc: dict, name: str = "relurax") -> ReluraxConfig:
    """ReluraxConfig from a checkpoint's config.json contents."""
    specs: list[DecoderLayerSpec] = []
    for i, lay in enumerate(hc["layers"]):
        m, f, kind = lay["mixer"], lay.get("mlp"), lay["type"]
        if kind == "attention":
            _heads(i, m, int(m["dim"]))
            mixer = AttentionSpec(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                                  scale=float(m["scale"]), conv=int(m["conv"]), window=int((m.get("mask") or {}).get("size", 0)))
            if mixer.kv_heads < 1 or mixer.heads % mixer.kv_heads:
                raise ValueError(f"layer {i}: {mixer.heads} query heads over {mixer.kv_heads} kv heads")
            if mixer.vdim != mixer.dim:
                raise ValueError(f"layer {i}: values are the keys, but their sizes are {mixer.vdim} and {mixer.dim}")
            if not 1 <= mixer.conv <= 8:
                raise ValueError(f"layer {i}: a convolution of {mixer.conv} taps (1..8 supported)")
            if "mask" in m and mixer.window < 1:
                raise ValueError(f"layer {i}: a window of {mixer.window} tokens")
        elif kind == "latent_attention":
            _heads(i, m, int(m["dim"]) + int(m["rot_dim"]))
            mixer = LatentSpec(heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=int(m["rot_dim"]), vdim=int(m["vdim"]),
                               q_rank=int(m["q_rank"]), kv_rank=int(m["kv_rank"]), scale=float(m["scale"]),
                               rot_base=float(m["rot"]["base"]), kv_from=-1 if m.get("kv_from") is None else int(m["kv_from"]))
            if mixer.rot_dim % 2 or int(m["rot"]["dims"]) != mixer.rot_dim:
                raise ValueError(f"layer {i}: {m['rot']['dims']} rotated dimensions of a part of {mixer.rot_dim}")
            if -(-mixer.kv_rank // 32) * 32 + mixer.rot_dim > 640 or mixer.q_rank > 4096:
                raise ValueError(f"layer {i}: latent sizes {mixer.q_rank} and {mixer.kv_rank} + {mixer.rot_dim}; "
                                 "the latent kernels go up to 4096 and 640")
            if mixer.kv_from >= 0:
                src = specs[mixer.kv_from].mixer if mixer.kv_from < i else None
                if not isinstance(src, LatentSpec) or src.kv_from >= 0 or (src.kv_rank, src.rot_dim, src.rot_base) != (
                        mixer.kv_rank, mixer.rot_dim, mixer.rot_base):
                    raise ValueError(f"layer {i}: layer {mixer.kv_from} keeps no latent rows of its kind")
        else:
            raise ValueError(f"layer {i}: mixer type {kind!r} not supported")
        if f is not None and f["kind"] != "dense":
            raise ValueError(f"layer {i}: feed-forward kind {f['kind']!r} not supported")
        specs.append(DecoderLayerSpec(mixer, None if f is None else FeedForwardSpec(int(f["ff"]))))
    if not specs:
        raise ValueError("no layers")
    return ReluraxConfig(name=name, vocab_size=int(hc["vocab"]), hidden=int(hc["width"]), rms_eps=float(hc["norm"]["eps"]),
                         layer_specs=tuple(specs))


# config.json "architecture" -> reader
DESIGNS = {"sufolix": sufolix_from_dict, "relurax": relurax_from_dict}


def config_from_dir(path: str, name: str | None = None) -> "LlamaConfig | SufolixConfig | ReluraxConfig":
    """The configuration a checkpoint directory's config.json describes, whichever of the
    supported architectures it is (``architecture``: a design of its own; ``model_type``: a
    HuggingFace Llama-architecture checkpoint)."""
    with open(os.path.join(path, "config.json")) as f:
        hc = json.load(f)
    arch = hc.get("architecture")
    if arch is None:
        return config_from_hf(path, name)
    if str(arch).lower() not in DESIGNS:
        raise ValueError(f"{path}: architecture {arch!r} not supported")
    return DESIGNS[str(arch).lower()](hc, name or os.path.basename(os.path.normpath(path)))
