"""Zazerax, written out plainly: one function per mechanism, float64, whole sequences, no cache.

The oracle of the Zazerax tests.  It shares nothing with the package: weights come in as a dict name -> tensor
([out, in] matrices), the configuration as the dict that config.json holds.

A sublayer reads the stream as it is, and its output is normed before it joins:
    x += LN1(mixer(x));  x += LN2(ff(x))          LN(y) = (y - mean) / sqrt(var + eps) * w
The mixer is grouped-query attention under a window (norms over the whole q and k projections, no rotation, a learned
bias per head and bucket of distance, one added to the softmax's denominator), or latent attention (keys and values from
a low-rank latent, one rotated key part for all heads) in two kinds: queries straight from the stream, a rotation that
pairs the halves of the rotated part with stretched frequencies, a gate per output element; or queries through a latent
of their own, adjacent pairs, a gate per head.  The feed-forward squares a relu.  An entry of the layer list may use
another entry's weights.
"""
from __future__ import annotations

import math

import numpy as np
import torch

F64 = torch.float64


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def visible(n: int, size: int | None = None):
    """[n, n] bool: query i (row) sees key j (column) if j <= i and, with a window, i - j < size."""
    dist = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    return (dist >= 0) & (dist < size) if size else dist >= 0


# --------------------------------------------------------------------------
# attention with a bias per bucket of distance
# --------------------------------------------------------------------------
def bucket(distance: int, rows: int, far: int) -> int:
    """Row of the bias table for a key `distance` back: the first rows // 2 distances have a row each, the others share
    rows that widen with the logarithm of the distance; from `far` on it is the last row.  Row half + k begins at
    half * (far / half)^(k / (rows - half)), compared in whole numbers."""
    half = rows // 2
    if distance < half:
        return distance
    k = 0
    while half + k < rows - 1 and distance ** (rows - half) * half ** (k + 1) >= far ** (k + 1) * half ** (rows - half):
        k += 1
    return half + k


def softmax_plus_one(s):
    """exp(s) / (1 + sum exp(s)) along the last dimension; masked entries are -inf."""
    top = torch.clamp(s.max(-1, keepdim=True).values, min=0.0)
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(-top))


def biased_attention(h, w, m, eps):
    n = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(h @ w["q"].T, w["q.norm"], eps).view(n, H, D)
    k = rms_norm(h @ w["k"].T, w["k.norm"], eps).view(n, G, D)
    v = (h @ w["v"].T).view(n, G, V)
    see = visible(n, (m.get("mask") or {}).get("size"))
    by_distance = torch.stack([w["rel"][bucket(d, w["rel"].shape[0], m["bias_max"])] for d in range(n)])      # [n, H]
    dist = (torch.arange(n)[:, None] - torch.arange(n)[None, :]).clamp(min=0)
    out = torch.zeros(n, H, V, dtype=h.dtype)
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * m["scale"] + by_distance[dist, a]
        out[:, a] = softmax_plus_one(s.masked_fill(~see, -math.inf)) @ v[:, g]
    return out.reshape(n, H * V) @ w["o"].T


# --------------------------------------------------------------------------
# rotations and latent attention
# --------------------------------------------------------------------------
def rotation(rot: dict):
    """(frequencies base^(-2i/dims), magnitude 1), or with `scaling` {factor, original, fast, slow}: pairs up to the one
    that turns `fast` times over `original` positions keep their frequency, those from the one that turns `slow` times
    on get it divided by `factor`, a ramp by index between; magnitude 0.1 ln(factor) + 1."""
    dims, base = rot["dims"], float(rot["base"])
    freqs = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return freqs, 1.0

    def index_of(turns):
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(index_of(sc["fast"])), 0)
    hi = min(math.ceil(index_of(sc["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freqs):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / sc["factor"] * ramp + f * (1.0 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate(vec, freqs, magnitude, halves: bool, angles: str = "float32"):
    """vec [n, ..., d], row t at position t: pair i of the first 2 len(freqs) entries, (i, i + len) with `halves`, else
    (2i, 2i + 1), turns by t f_i and grows by `magnitude`.  angles="float32": frequency and product rounded to float32,
    as a 32-bit implementation has them; "exact": float64."""
    out = vec.clone()
    for i, f in enumerate(freqs):
        a, b = (i, i + len(freqs)) if halves else (2 * i, 2 * i + 1)
        for t in range(vec.shape[0]):
            x = float(np.float32(t) * np.float32(f)) if angles == "float32" else t * f
            c, s = math.cos(x) * magnitude, math.sin(x) * magnitude
            u, v = vec[t, ..., a], vec[t, ..., b]
            out[t, ..., a] = u * c - v * s
            out[t, ..., b] = v * c + u * s
    return out


def latent_attention(h, w, m, eps, halves: bool, gate: str, angles: str = "float32"):
    """`gate` "element": a gate per output element; "head": one per head.  Queries go through a latent where the layer
    has tensors for one ('dq')."""
    n = h.shape[0]
    H, D, P, V, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    freqs, mag = rotation(m["rot"])
    q = rms_norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T if "dq" in w else h @ w["q"].T
    q = q.view(n, H, D + P)
    down = h @ w["dkv"].T
    c = rms_norm(down[:, :R], w["dkv.norm"], eps)
    k_rot = rotate(down[:, R:], freqs, mag, halves, angles)
    q_rot = rotate(q[..., D:], freqs, mag, halves, angles)
    k, v = (c @ w["uk"].T).view(n, H, D), (c @ w["uv"].T).view(n, H, V)
    see = visible(n)
    out = torch.zeros(n, H, V, dtype=h.dtype)
    for a in range(H):
        s = (q[:, a, :D] @ k[:, a].T + q_rot[:, a] @ k_rot.T) * m["scale"]
        out[:, a] = torch.softmax(s.masked_fill(~see, -math.inf), dim=-1) @ v[:, a]
    g = torch.sigmoid(h @ w["g"].T)
    out = out * g.unsqueeze(-1) if gate == "head" else out * g.view(n, H, V)
    return out.reshape(n, H * V) @ w["o"].T


MIXERS = {
    "attention": lambda h, w, m, eps, angles: biased_attention(h, w, m, eps),
    "latent_attention": lambda h, w, m, eps, angles: latent_attention(h, w, m, eps, True, "element", angles),
    "latent_attention_2": lambda h, w, m, eps, angles: latent_attention(h, w, m, eps, False, "head", angles),
}


# --------------------------------------------------------------------------
# feed-forward and the model
# --------------------------------------------------------------------------
def squared_relu_mlp(h, w):
    return torch.clamp(h @ w["up"].T, min=0.0) ** 2 @ w["down"].T


def sub(weights: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg: dict, weights: dict, tokens: list, dtype=F64, angles: str = "float32", layers_out=None):
    """Logits [n, vocab] of one sequence from position 0.  `layers_out`: a list that receives the stream after every
    layer.  (A test that wants a mechanism left out changes the configuration or the weights.)"""
    W = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.tensor(tokens)] * (cfg.get("embedding") or {}).get("scale", 1.0)
    for i, layer in enumerate(cfg["layers"]):
        owner = i
        while cfg["layers"][owner].get("weights_of") is not None:
            owner = cfg["layers"][owner]["weights_of"]
        w, m = sub(W, f"l{owner}."), layer["mixer"]
        x = x + layer_norm(MIXERS[layer["type"]](x, sub(w, "mix."), m, eps, angles), w["norm1"], eps)
        if layer.get("mlp"):
            x = x + layer_norm(squared_relu_mlp(x, sub(w, "mlp.")), w["norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return layer_norm(x, W["final.norm"], eps) @ W["head"].T
