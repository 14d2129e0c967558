"""Plain, slow implementation of the Sufolix decoder for the tests (one function per
mechanism, fp64 or fp32 on the CPU, whole sequences, no cache and no batching).

It shares nothing with ``operator_amd``: ``cfg`` is the dict of a config.json and ``w`` a dict
of CPU tensors under the checkpoint's names. A sequence is a list of token ids; every function
takes and returns [tokens, ...] tensors.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps, weight=None):
    """x / sqrt(mean(x^2) + eps), optionally scaled per feature."""
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def rotate(x, positions, base, dims):
    """Rotary positions on the first ``dims`` features of [tokens, heads, dim], neighbours paired
    (0 with 1, 2 with 3, ...); pair i turns by position * base^(-2 i / dims)."""
    y = x.clone()
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        for t, p in enumerate(positions):
            a = float(p) * f
            c, s = math.cos(a), math.sin(a)
            u, v = x[t, :, 2 * i], x[t, :, 2 * i + 1]
            y[t, :, 2 * i] = u * c - v * s
            y[t, :, 2 * i + 1] = v * c + u * s
    return y


def mix_values(v, v_first, lam):
    return (1.0 - lam) * v + lam * v_first


def attend(q, k, v, scale):
    """Causal softmax attention: q [T, H, D], k [T, G, D], v [T, G, Dv]; query head h reads
    key/value head h // (H / G)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    mask = torch.ones(T, T, dtype=torch.bool).triu(1)
    for h in range(H):
        g = h // per
        s = (q[:, h] @ k[:, g].T) * scale
        s = s.masked_fill(mask, float("-inf"))
        out[:, h] = torch.softmax(s, -1) @ v[:, g]
    return out


def qkv(h, w, pre, m, eps):
    """Projected, biased, rotated and normalised q, k and the unmixed v of one layer."""
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ w[pre + "q"].T + w[pre + "q.b"]).view(T, H, D)
    k = (h @ w[pre + "k"].T + w[pre + "k.b"]).view(T, G, D)
    v = (h @ w[pre + "v"].T + w[pre + "v.b"]).view(T, G, Dv)
    pos = range(T)
    q = rms(rotate(q, pos, m["rot"]["base"], m["rot"]["dims"]), eps)
    k = rms(rotate(k, pos, m["rot"]["base"], m["rot"]["dims"]), eps)
    return q, k, v


def attention(h, w, pre, m, eps, first):
    """The attention mixer; ``first`` is a dict that carries the first mixing layer's values."""
    q, k, v = qkv(h, w, pre, m, eps)
    if m.get("v_mix"):
        if "v" in first:
            v = mix_values(v, first["v"], w[pre + "vmix"].reshape(()))
        else:
            first["v"] = v
    o = attend(q, k, v, m["scale"])
    return o.reshape(h.shape[0], -1) @ w[pre + "o"].T


def gated(h, w, pre):
    g, u = h @ w[pre + "gate"].T, h @ w[pre + "up"].T
    return (g * torch.sigmoid(g) * u) @ w[pre + "down"].T


def route(h, w, pre, router, close=None):
    """(expert ids, weights) [T, top]: the largest sigmoid scores, used as they are. ``close``: a
    list that receives, per token, the gap between the last expert taken and the first one left,
    relative to the spread of the logits."""
    z = h @ w[pre + "router"].T
    s = torch.sigmoid(z)
    val, idx = torch.topk(s, router["top"], dim=-1)
    if close is not None and router["top"] < router["experts"]:
        v = torch.sort(z, dim=-1, descending=True)[0]
        close.append((v[:, router["top"] - 1] - v[:, router["top"]]) / z.std())
    return idx, val


def experts(h, w, pre, c, close=None):
    idx, val = route(h, w, pre, c["router"], close)
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(idx[t].tolist(), val[t]):
            y[t] += gated((s * h[t]).unsqueeze(0), w, f"{pre}e{e}.")[0]
    if c.get("shared"):
        y = y + torch.sigmoid(h @ w[pre + "shared.sg"].T) * gated(h, w, pre + "shared.")
    return y


def sublayer_in(xs, w, pre):
    """[T, S, width] streams -> the sublayer's input."""
    return torch.einsum("tsw,s->tw", xs, w[pre + "in"])


def sublayer_out(xs, y, w, pre):
    """New streams from the old ones and the sublayer's output (mix is [from, to])."""
    return torch.einsum("tsw,sr->trw", xs, w[pre + "mix"]) + w[pre + "out"][None, :, None] * y[:, None, :]


def forward(cfg, w, tokens, dtype=torch.float64, layer_out=None, close=None):
    """Logits [T, vocab] of one sequence; ``layer_out``: a list that receives the stream sum
    after every layer; ``close``: one that receives every router's gaps (``route``)."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    xs = x[:, None, :].repeat(1, cfg["streams"], 1)
    first: dict = {}
    for i, lay in enumerate(cfg["layers"]):
        pre = f"l{i}."
        u = rms(sublayer_in(xs, w, pre + "hc1."), eps, w[pre + "norm1"])
        xs = sublayer_out(xs, attention(u, w, pre + "mix.", lay["mixer"], eps, first), w, pre + "hc1.")
        if lay.get("mlp") is not None:
            u = rms(sublayer_in(xs, w, pre + "hc2."), eps, w[pre + "norm2"])
            y = gated(u, w, pre + "mlp.") if lay["mlp"]["kind"] == "dense" else experts(u, w, pre + "mlp.", lay["mlp"], close)
            xs = sublayer_out(xs, y, w, pre + "hc2.")
        if layer_out is not None:
            layer_out.append(xs.sum(1))
    return rms(xs.sum(1), eps, w["final.norm"]) @ w["head"].T
