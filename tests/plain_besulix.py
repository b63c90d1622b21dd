"""Plain, slow Besulix: every formula of the design, one function per mechanism, float64 on the CPU, whole sequences
at once, no cache.  It shares no code with the package: tests hold the engine against it.

A model is (cfg, w): cfg the config.json dict, w a dict name -> float64 tensor.  `forward(cfg, w, tokens)` returns
logits [T, vocab]; `layers_out` receives the stream after every layer."""
from __future__ import annotations

import math

import torch


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def logsigmoid(x):
    return torch.where(x < -30.0, x, -torch.log1p(torch.exp(-torch.clamp(x, min=-30.0))))


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, weight, eps):
    return unit_rms(x, eps) * weight


def turn(x, positions, base, sign=1.0):
    """x [T, heads, dims] with the pairs (m, m + dims/2) turned by sign * position * base^(-2m/dims)."""
    n = x.shape[-1]
    freq = torch.tensor([base ** (-2.0 * m / n) for m in range(n // 2)], dtype=x.dtype)
    angle = sign * positions.to(x.dtype)[:, None, None] * freq
    c, s = torch.cos(angle), torch.sin(angle)
    u, v = x[..., :n // 2], x[..., n // 2:]
    return torch.cat([u * c - v * s, v * c + u * s], dim=-1)


def rotary(x, positions, base, dims):
    """The first `dims` dimensions of every head turned, the rest as they are."""
    return torch.cat([turn(x[..., :dims], positions, base), x[..., dims:]], dim=-1)


def chunk_visible(T, size):
    """[query, key]: keys up to the query's own position, in the query's own chunk."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & (i // size == j // size)


def softmax_with_sink(scores, visible, sink):
    """Rows of weights over the visible keys; exp(sink) joins the denominator and goes nowhere."""
    s = torch.where(visible, scores, torch.full_like(scores, -math.inf))
    top = torch.clamp(s.max(-1, keepdim=True).values, min=float(sink))
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def chunked_attention(h, w, p, m):
    """Grouped-query attention inside chunks: rotated keys and queries, rotated values turned back at the query, a
    temperature and a sink per head."""
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    pos = torch.arange(T)
    q = (h @ w[p + "q"].T + w[p + "q.b"]).view(T, H, D)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).view(T, G, D)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).view(T, G, V)
    base, dims = m["rot"]["base"], m["rot"]["dims"]
    q, k = rotary(q, pos, base, dims), rotary(k, pos, base, dims)
    v = turn(v, pos, base)
    visible = chunk_visible(T, m["mask"]["size"])
    outs = []
    for head in range(H):
        g = head // (H // G)
        scores = (q[:, head] @ k[:, g].T) * m["scale"] * w[p + "temp"][head]
        outs.append(softmax_with_sink(scores, visible, w[p + "sink"][head]) @ v[:, g])
    o = turn(torch.stack(outs, dim=1), pos, base, sign=-1.0)
    return o.reshape(T, H * V) @ w[p + "o"].T


def shifted(h):
    """The token before; zeros before the first."""
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]], dim=0)


def channel_decay(mix, w, p):
    """The factor a key channel of the state is multiplied by at this token."""
    return torch.exp(-torch.exp(torch.tanh(mix @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]))


def time_mix(h, w, p, m, eps):
    """A linear recurrence with a decay per token and channel and a bonus for the current token, read by mixes of the
    token and the one before it."""
    H, D = m["heads"], m["dim"]
    T = h.shape[0]
    delta = shifted(h) - h
    mixes = {s: h + delta * w[p + "mu." + s] for s in "rkvgw"}
    r, k, v = ((mixes[s] @ w[p + s].T).view(T, H, D) for s in "rkv")
    gate = silu(mixes["g"] @ w[p + "g"].T)
    decay = channel_decay(mixes["w"], w, p).view(T, H, D)
    bonus = w[p + "u"].view(H, D)
    S = torch.zeros(H, D, D, dtype=h.dtype)
    out = []
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out.append(torch.einsum("hdv,hd->hv", S + bonus[:, :, None] * kv, r[t]))
        S = decay[t][:, :, None] * S + kv
    o = unit_rms(torch.stack(out), eps).reshape(T, H * D) * w[p + "norm"]
    return (o * gate) @ w[p + "o"].T


def side_by_side(h, w, p, m, eps):
    return m["left_scale"] * chunked_attention(h, w, p + "left.", m["left"]) \
        + m["right_scale"] * time_mix(h, w, p + "right.", m["right"], eps)


def matrix_memory(h, w, p, m, eps):
    """A matrix memory with exponential gates kept in range by a running maximum that starts at zero."""
    H, D, V, cap = m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    T = h.shape[0]
    q = (h @ w[p + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ w[p + "k"].T).view(T, H, D)
    v = (h @ w[p + "v"].T).view(T, H, V)
    i_gate = cap * torch.tanh((h @ w[p + "i"].T + w[p + "i.b"]) / cap)
    f_gate = logsigmoid(cap * torch.tanh((h @ w[p + "f"].T + w[p + "f.b"]) / cap))
    S = torch.zeros(H, D, V, dtype=h.dtype)
    n = torch.zeros(H, D, dtype=h.dtype)
    top = torch.zeros(H, dtype=h.dtype)
    out = []
    for t in range(T):
        new = torch.maximum(f_gate[t] + top, i_gate[t])
        keep, take = torch.exp(f_gate[t] + top - new), torch.exp(i_gate[t] - new)
        S = keep[:, None, None] * S + take[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + take[:, None] * k[t]
        top = new
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-top)) + 1e-6
        out.append(torch.einsum("hdv,hd->hv", S, q[t]) / den[:, None])
    o = unit_rms(torch.stack(out), eps).reshape(T, H * V) * w[p + "norm"]
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def clamped_ff(h, w, p, limit):
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def mixer(kind, h, w, p, m, eps):
    return {"parallel": side_by_side, "mlstm": matrix_memory}[kind](h, w, p, m, eps)


def layer(x, w, i, entry, eps):
    lp = f"l{i}."
    x = x + mixer(entry["type"], rms_norm(x, w[lp + "norm1"], eps), w, lp + "mix.", entry["mixer"], eps)
    if entry.get("mlp") is None:
        return x
    return x + clamped_ff(rms_norm(x, w[lp + "norm2"], eps), w, lp + "mlp.", entry["mlp"]["limit"])


def capped(logits, cap):
    return cap * torch.tanh(logits / cap)


def embed(cfg, w, tokens):
    return rms_norm(w["embed"][torch.as_tensor(tokens, dtype=torch.int64)], w["embed.norm"], cfg["norm"]["eps"])


def forward(cfg, w, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence from position 0."""
    eps = cfg["norm"]["eps"]
    x = embed(cfg, w, tokens)
    for i, entry in enumerate(cfg["layers"]):
        x = layer(x, w, i, entry, eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return capped(rms_norm(x, w["final.norm"], eps) @ w["head"].T, cfg["logit_softcap"])
