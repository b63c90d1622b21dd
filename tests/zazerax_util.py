"""Helpers of the Zazerax tests: small configurations, weights made in the test, and the comparison of the
engine's logits with the plain model (`plain_zazerax`)."""
from __future__ import annotations

import copy

import torch

import plain_zazerax as plain
from rafilix_util import random_tokens, row_errors, run_schedule, write_model  # noqa: F401  (schedules and files are alike)

STRETCH = (3.0, 40, 4.0, 0.5)        # (factor, original, fast, slow): with base 100 and 8 rotated dimensions all three bands occur
BIAS_ROWS = 12                       # rows of the distance biases where a test does not say


def attention_layer(heads=4, kv_heads=2, dim=16, vdim=16, scale=0.3, bias_max=20, window=13, mlp=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "bias_max": bias_max}
    if window:
        mixer["mask"] = {"size": window}
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def latent_layer(heads=4, dim=16, rot_dim=8, vdim=24, kv_rank=32, scale=0.3, base=100.0, scaling=STRETCH, q_rank=None,
                 rot_dims=None, mlp=None):
    """Without `q_rank` the kind whose queries come straight from the stream; `rot_dims` None: all of rot_dim is turned."""
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
             "rot": {"base": base, "dims": rot_dim if rot_dims is None else rot_dims}}
    if scaling:
        mixer["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if q_rank:
        mixer["q_rank"] = q_rank
    return {"type": "latent_attention_2" if q_rank else "latent_attention", "mixer": mixer, "mlp": mlp}


def latent_layer_2(**kw):
    return latent_layer(**{"q_rank": 20, "scaling": None, **kw})


def again(layers: list, j: int) -> dict:
    """A layer that runs layer j's weights."""
    return {**copy.deepcopy(layers[j]), "weights_of": j}


def dense(ff=48):
    return {"kind": "dense", "ff": ff}


def config(layers, width=64, vocab=160, eps=1e-6, emb_scale=1.7):
    out = {"architecture": "Zazerax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if emb_scale is not None:
        out["embedding"] = {"scale": emb_scale}
    return out


def _main_layers():
    """Layers unlike each other: windows of 13, 5 and 30, one wider than the distance at which the biases' last row begins,
    key heads as many as query heads and one for all, value heads narrower and wider than key heads; both kinds of latent
    attention with stretched and plain frequencies, with fewer turned dimensions than the rotated part has; layers without a
    feed-forward; two entries that run an earlier entry's weights, one of them a windowed one."""
    layers = [
        attention_layer(heads=4, kv_heads=2, dim=16, vdim=24, scale=0.35, bias_max=20, window=13, mlp=dense(48)),
        latent_layer(heads=3, dim=16, rot_dim=8, vdim=24, kv_rank=24, scale=0.35, mlp=dense(40)),
        latent_layer_2(heads=5, dim=8, rot_dim=12, vdim=16, kv_rank=20, q_rank=28, scale=0.4, rot_dims=8, base=50.0, mlp=None),
        attention_layer(heads=3, kv_heads=3, dim=24, vdim=16, scale=0.3, bias_max=14, window=30, mlp=dense(24)),
    ]
    layers.append(again(layers, 1))
    layers.append(again(layers, 0))
    layers.append(latent_layer(heads=2, dim=24, rot_dim=12, vdim=8, kv_rank=16, scale=0.3, base=300.0, scaling=None, mlp=dense(16)))
    layers.append(attention_layer(heads=5, kv_heads=1, dim=8, vdim=8, scale=0.5, bias_max=30, window=5, mlp=None))
    return layers


CFG_MAIN = config(_main_layers())
# bfloat16 on the matrix units: sizes in multiples of 16, widths in multiples of 64
CFG_MFMA = config([
    attention_layer(heads=4, kv_heads=2, dim=64, vdim=64, scale=0.2, bias_max=60, window=100, mlp=dense(128)),
    latent_layer(heads=4, dim=32, rot_dim=16, vdim=32, kv_rank=64, scale=0.2, base=1000.0, scaling=(2.0, 64, 8.0, 1.0), mlp=dense(192)),
    latent_layer_2(heads=2, dim=64, rot_dim=32, vdim=64, kv_rank=96, q_rank=64, scale=0.15, base=1000.0, mlp=dense(64)),
    attention_layer(heads=2, kv_heads=1, dim=128, vdim=128, scale=0.15, bias_max=200, window=150, mlp=None),
], width=128, vocab=256)


def tensor_shapes(cfg: dict, bias_rows: int = BIAS_ROWS) -> dict:
    """Names and shapes of a model's tensors, from its configuration."""
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "final.norm": (W,), "head": (cfg["vocab"], W)}
    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p, m = f"l{i}.", layer["mixer"]
        H, D, V = m["heads"], m["dim"], m["vdim"]
        out[p + "norm1"] = (W,)
        if layer["type"] == "attention":
            G = m["kv_heads"]
            out.update({p + "mix.q": (H * D, W), p + "mix.k": (G * D, W), p + "mix.v": (G * V, W), p + "mix.q.norm": (H * D,),
                        p + "mix.k.norm": (G * D,), p + "mix.rel": (bias_rows, H), p + "mix.o": (W, H * V)})
        else:
            P, R = m["rot_dim"], m["kv_rank"]
            out.update({p + "mix.dkv": (R + P, W), p + "mix.dkv.norm": (R,), p + "mix.uk": (H * D, R), p + "mix.uv": (H * V, R),
                        p + "mix.o": (W, H * V)})
            if layer["type"] == "latent_attention":
                out.update({p + "mix.q": (H * (D + P), W), p + "mix.g": (H * V, W)})
            else:
                Rq = m["q_rank"]
                out.update({p + "mix.dq": (Rq, W), p + "mix.dq.norm": (Rq,), p + "mix.uq": (H * (D + P), Rq), p + "mix.g": (H, W)})
        if layer.get("mlp"):
            out.update({p + "norm2": (W,), p + "mlp.up": (layer["mlp"]["ff"], W), p + "mlp.down": (W, layer["mlp"]["ff"])})
    return out


def make_weights(cfg: dict, seed: int, bias_rows: int = BIAS_ROWS) -> dict:
    """Random weights, bfloat16 values: a missing key, a wrong row of the biases or a sink that is left out moves the logits."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, bias_rows).items():
        last = name.split(".")[-1]
        if last.startswith("norm"):
            t = 1.0 + 0.2 * torch.randn(shape, generator=gen)
            if last in ("norm1", "norm2"):      # behind a sublayer: half the stream's size, or eight layers multiply every rounding
                t = 0.5 * t
        elif last == "rel":
            t = 1.2 * torch.randn(shape, generator=gen)
        elif name == "embed":
            t = torch.randn(shape, generator=gen) / (cfg.get("embedding") or {}).get("scale", 1.0)
        else:
            t = 1.3 * torch.randn(shape, generator=gen) / shape[-1] ** 0.5
        out[name] = t.to(torch.bfloat16)
    return out


def as_float64(weights: dict) -> dict:
    return {k: v.to(torch.float64) for k, v in weights.items()}


# (float32 is the sharp test.  bfloat16: every sublayer's output is normed to the size of a row before it joins, so its
# roundings weigh as much as the sublayer itself.  EDGE_LIMIT: for models with peaked softmaxes, whose rounding errors are
# larger, and for one engine run against another.)
LIMIT = {"float32": 2e-5, "bfloat16": 6e-2}
EDGE_LIMIT = {"float32": 6e-5, "bfloat16": 1e-1}


def check_against_plain(cfg, weights, requests, got, dtype, what="", limit=None):
    """Every position of every request against the plain model."""
    limit = limit or LIMIT[dtype]
    worst = 0.0
    for r, tokens in requests.items():
        err = row_errors(got[r], plain.forward(cfg, weights, tokens))
        i = int(err.argmax())
        assert float(err[i]) <= limit, (f"{what} request {r}: position {i} of {len(tokens)} is off by {float(err[i]):.3g} "
                                        f"(limit {limit:g}); first position over it: {int((err > limit).nonzero()[0])}")
        worst = max(worst, float(err[i]))
    return worst


def changed(cfg: dict, layer: int, **mixer_changes) -> dict:
    """The configuration with keys of one layer's mixer replaced (None takes a key out), in the entries that run its
    weights too."""
    out = copy.deepcopy(cfg)
    for i, entry in enumerate(out["layers"]):
        if i == layer or entry.get("weights_of") == layer:
            for key, value in mixer_changes.items():
                if value is None:
                    entry["mixer"].pop(key, None)
                else:
                    entry["mixer"][key] = value
    return out
