"""Helpers of the Besulix tests: small configurations, weights made in the test, and the comparison of the engine's
logits with the plain model (`plain_besulix`)."""
from __future__ import annotations

import copy

import torch

import plain_besulix as plain
from rafilix_util import random_tokens, row_errors, run_schedule, write_model  # noqa: F401  (schedules and files are alike)


def parallel_layer(heads=4, kv_heads=2, dim=16, vdim=12, scale=0.3, base=10000.0, dims=8, chunk=24, r_heads=3, r_dim=8, left=0.7,
                   right=1.1, mlp=None):
    return {"type": "parallel", "mlp": mlp, "mixer": {
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"base": base, "dims": dims},
                 "mask": {"size": chunk}},
        "right": {"heads": r_heads, "dim": r_dim}, "left_scale": left, "right_scale": right}}


def mlstm_layer(heads=3, dim=8, vdim=12, gate_cap=10.0, mlp=None):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}, "mlp": mlp}


def dense(ff=40, limit=1.2):
    return {"kind": "dense", "ff": ff, "limit": limit}


def config(layers, width=48, vocab=150, eps=1e-5, softcap=6.0):
    return {"architecture": "Besulix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_softcap": softcap, "layers": layers}


# Layers unlike each other, in an order of their own: both mixers several times with other sizes, with and without a
# feed-forward, partial and whole rotations, chunks of 7, 24 and 50 positions (cache groups of their own), heads that
# share key heads and heads that do not, values narrower and wider than keys, scales of both signs and one of 1.
CFG_MAIN = config([
    mlstm_layer(heads=3, dim=8, vdim=12, gate_cap=10.0, mlp=dense(40, 1.2)),
    parallel_layer(heads=4, kv_heads=2, dim=16, vdim=12, scale=0.3, dims=8, chunk=24, r_heads=3, r_dim=8, left=0.7, right=1.1,
                   mlp=dense(24, 0.6)),
    parallel_layer(heads=3, kv_heads=3, dim=12, vdim=20, scale=0.45, base=500.0, dims=12, chunk=7, r_heads=2, r_dim=20, left=1.0,
                   right=-0.8, mlp=None),
    mlstm_layer(heads=2, dim=20, vdim=8, gate_cap=4.0, mlp=None),
    parallel_layer(heads=2, kv_heads=1, dim=24, vdim=24, scale=0.25, base=100.0, dims=4, chunk=50, r_heads=1, r_dim=32, left=1.2,
                   right=0.5, mlp=dense(56, 3.0)),
], width=48, vocab=150, softcap=5.0)
# bfloat16 on the matrix units: sizes in multiples of 16, widths in multiples of 64; value heads of the keys' size,
# narrower ones, and heads wider than 128
CFG_MFMA = config([
    parallel_layer(heads=4, kv_heads=2, dim=64, vdim=64, scale=0.15, dims=32, chunk=80, r_heads=4, r_dim=32, mlp=dense(128, 2.0)),
    mlstm_layer(heads=2, dim=64, vdim=32, gate_cap=12.0, mlp=None),
    parallel_layer(heads=2, kv_heads=1, dim=128, vdim=48, scale=0.1, dims=128, chunk=150, r_heads=2, r_dim=64, left=0.9, right=0.7,
                   mlp=dense(64, 1.0)),
    parallel_layer(heads=3, kv_heads=3, dim=160, vdim=96, scale=0.08, dims=96, chunk=100, r_heads=2, r_dim=128, left=0.8, right=0.6),
    parallel_layer(heads=2, kv_heads=2, dim=128, vdim=128, scale=0.1, dims=64, chunk=200, r_heads=3, r_dim=16, left=0.6, right=0.8),
], width=128, vocab=256, softcap=8.0)
DECAY_RANK = 5


def tensor_shapes(cfg: dict, decay_rank: int = DECAY_RANK) -> dict:
    """Names and shapes of a model's tensors, from its configuration."""
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "embed.norm": (W,), "final.norm": (W,), "head": (cfg["vocab"], W)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        out[p + "norm1"] = (W,)
        q = p + "mix."
        if layer["type"] == "mlstm":
            H, D, V = m["heads"], m["dim"], m["vdim"]
            out.update({q + "q": (H * D, W), q + "k": (H * D, W), q + "v": (H * V, W), q + "g": (H * V, W), q + "i": (H, W),
                        q + "i.b": (H,), q + "f": (H, W), q + "f.b": (H,), q + "norm": (H * V,), q + "o": (W, H * V)})
        else:
            a, b = m["left"], m["right"]
            H, G, D, V = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            for name, rows in (("q", H * D), ("k", G * D), ("v", G * V)):
                out.update({q + f"left.{name}": (rows, W), q + f"left.{name}.b": (rows,)})
            out.update({q + "left.temp": (H,), q + "left.sink": (H,), q + "left.o": (W, H * V)})
            I = b["heads"] * b["dim"]
            for name in "rkvg":
                out[q + f"right.{name}"] = (I, W)
            for name in "rkvgw":
                out[q + f"right.mu.{name}"] = (W,)
            out.update({q + "right.w1": (decay_rank, W), q + "right.w2": (I, decay_rank), q + "right.w0": (I,),
                        q + "right.u": (b["heads"], b["dim"]), q + "right.norm": (I,), q + "right.o": (W, I)})
        f = layer.get("mlp")
        if f:
            out.update({p + "norm2": (W,), p + "mlp.gate": (f["ff"], W), p + "mlp.up": (f["ff"], W), p + "mlp.down": (W, f["ff"])})
    return out


def make_weights(cfg: dict, seed: int, decay_rank: int = DECAY_RANK) -> dict:
    """Random weights, bfloat16 values, of a size that keeps every sublayer's output of order one: a lost state, a
    missing key, a sink or a mix that is left out then moves the logits."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, decay_rank).items():
        last = name.split(".")[-1]
        rand = torch.randn(shape, generator=gen)
        if name.endswith(".f.b"):
            t = 2.5 + 0.3 * rand                          # a memory that forgets slowly
        elif name.endswith(".b"):
            t = 0.3 * rand
        elif last in ("norm", "norm1", "norm2"):
            t = 1.0 + 0.2 * rand
        elif last == "temp":
            t = 1.0 + 0.4 * torch.rand(shape, generator=gen) * (1 if seed % 2 else -1)
        elif last == "sink":
            t = 1.5 + rand
        elif ".mu." in name:
            t = torch.rand(shape, generator=gen)
        elif last == "w0":
            t = -2.5 + rand                               # decays of 0.75 to 0.99
        elif last == "w2":
            t = 0.8 * rand
        elif last == "u":
            t = 0.7 * rand
        elif name == "embed":
            t = rand
        elif name == "head":
            t = 3.0 * rand / shape[-1] ** 0.5
        else:
            t = 1.3 * rand / shape[-1] ** 0.5
        out[name] = t.to(torch.bfloat16)
    return out


def as_float64(weights: dict) -> dict:
    return {k: v.to(torch.float64) for k, v in weights.items()}


LIMIT = {"float32": 3e-5, "bfloat16": 6e-2}
EDGE_LIMIT = {"float32": 6e-5, "bfloat16": 1e-1}


def check_against_plain(cfg, weights, requests, got, dtype, what="", limit=None):
    """Every position of every request against the plain model."""
    limit = limit or LIMIT[dtype]
    w64 = as_float64(weights)
    worst = 0.0
    for r, tokens in requests.items():
        err = row_errors(got[r], plain.forward(cfg, w64, tokens))
        i = int(err.argmax())
        assert float(err[i]) <= limit, (f"{what} request {r}: position {i} of {len(tokens)} is off by {float(err[i]):.3g} "
                                        f"(limit {limit:g}); first position over it: {int((err > limit).nonzero()[0])}")
        worst = max(worst, float(err[i]))
    return worst


def changed(cfg: dict, layer: int, **changes) -> dict:
    """The configuration with keys of one layer's mixer replaced ('left__scale' reaches into 'left')."""
    out = copy.deepcopy(cfg)
    for key, value in changes.items():
        at = out["layers"][layer]["mixer"]
        parts = key.split("__")
        for part in parts[:-1]:
            at = at[part]
        at[parts[-1]] = value
    return out
