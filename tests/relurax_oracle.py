"""Plain, slow implementation of the Relurax decoder for the tests (one function per mechanism,
fp64 or fp32 on the CPU, whole sequences, no cache and no batching).

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


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def short_conv(u, taps):
    """Causal convolution of every channel of u [T, C] with its own row of ``taps`` [C, n]; the
    last tap meets the current token, zeros come before the first one."""
    n = taps.shape[1]
    y = torch.zeros_like(u)
    for t in range(u.shape[0]):
        for j in range(n):
            s = t - (n - 1) + j
            if s >= 0:
                y[t] += taps[:, j] * u[s]
    return y


def rotate_half(x, positions, base):
    """All dims of x [tokens, heads, dims]: i turns with i + dims / 2 by position * base^(-2 i / dims)."""
    y, dims = x.clone(), x.shape[-1]
    n = dims // 2
    for i in range(n):
        f = base ** (-2.0 * i / dims)
        for t, p in enumerate(positions):
            c, s = math.cos(float(p) * f), math.sin(float(p) * f)
            u, v = x[t, :, i], x[t, :, i + n]
            y[t, :, i] = u * c - v * s
            y[t, :, i + n] = v * c + u * s
    return y


def attend(q, k, v, scale, window=None):
    """Softmax attention: q [T, H, D], k [T, G, D], v [T, G, Dv]; query head h reads key/value head
    h // (H / G); token i sees j <= i, with ``window`` only i - j < window."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    hidden = j > i
    if window is not None:
        hidden = hidden | (i - j >= window)
    for h in range(H):
        g = h // per
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(hidden, float("-inf"))
        out[:, h] = torch.softmax(s, -1) @ v[:, g]
    return out


def head_gate(o, h, w, pre):
    """Every head's output times its sigmoid gate, one number per head and token."""
    return o * torch.sigmoid(h @ w[pre + "g"].T)[..., None]


def attention_qkv(h, w, pre, m, eps):
    """Convolved and normalised q, k; the values are the convolved keys."""
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    T = h.shape[0]
    q = short_conv(h @ w[pre + "q"].T, w[pre + "q.conv"]).view(T, H, D)
    k = short_conv(h @ w[pre + "k"].T, w[pre + "k.conv"]).view(T, G, D)
    return rms(q, eps, w[pre + "q.norm"]), rms(k, eps, w[pre + "k.norm"]), k


def attention(h, w, pre, m, eps):
    q, k, v = attention_qkv(h, w, pre, m, eps)
    o = head_gate(attend(q, k, v, m["scale"], m["mask"]["size"]), h, w, pre)
    return o.reshape(h.shape[0], -1) @ w[pre + "o"].T


def latent(h, w, pre, m, eps):
    """What the layer caches: (c [T, kv_rank], the rotated key part [T, rot_dim])."""
    R = m["kv_rank"]
    z = h @ w[pre + "dkv"].T
    rot = rotate_half(z[:, None, R:], range(h.shape[0]), m["rot"]["base"])[:, 0]
    return rms(z[:, :R], eps, w[pre + "dkv.norm"]), rot


def latent_queries(h, w, pre, m, eps):
    """q [T, H, dim + rot_dim] with its last part rotated."""
    T, H, D = h.shape[0], m["heads"], m["dim"]
    q = (rms(h @ w[pre + "dq"].T, eps, w[pre + "dq.norm"]) @ w[pre + "uq"].T).view(T, H, D + m["rot_dim"])
    return torch.cat([q[..., :D], rotate_half(q[..., D:], range(T), m["rot"]["base"])], -1)


def latent_keys_values(c, rot, w, pre, m):
    T, H = c.shape[0], m["heads"]
    k = (c @ w[pre + "uk"].T).view(T, H, m["dim"])
    return torch.cat([k, rot[:, None].expand(T, H, -1)], -1), (c @ w[pre + "uv"].T).view(T, H, m["vdim"])


def latent_attention(h, w, pre, m, eps, kept):
    """``kept``: (c, rotated part) of this layer, or of the layer it reads."""
    k, v = latent_keys_values(*kept, w, pre, m)
    o = head_gate(attend(latent_queries(h, w, pre, m, eps), k, v, m["scale"]), h, w, pre)
    return o.reshape(h.shape[0], -1) @ w[pre + "o"].T


def gated(h, w, pre):
    return (gelu_tanh(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def forward(cfg, w, tokens, dtype=torch.float64, layer_out=None):
    """Logits [T, vocab] of one sequence; ``layer_out``: a list that receives the residual after
    every layer."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    kept: dict = {}
    for i, lay in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lay["mixer"]
        h = rms(x, eps, w[p + "norm1"])
        if lay["type"] == "attention":
            y = attention(h, w, p + "mix.", m, eps)
        else:
            src = m.get("kv_from", i)
            if src == i:
                kept[i] = latent(h, w, p + "mix.", m, eps)
            y = latent_attention(h, w, p + "mix.", m, eps, kept[src])
        x = x + rms(y, eps, w[p + "norm1b"])
        if lay.get("mlp") is not None:
            x = x + rms(gated(rms(x, eps, w[p + "norm2"]), w, p + "mlp."), eps, w[p + "norm2b"])
        if layer_out is not None:
            layer_out.append(x)
    return rms(x, eps, w["final.norm"]) @ w["head"].T
