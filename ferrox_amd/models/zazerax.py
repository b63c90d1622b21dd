"""Zazerax as a list of parts.

Every layer is a post-norm block, x += N1(mixer(x)), x += N2(ff(x)), N a layer norm without a bias; a layer may have no
feed-forward.  The mixer is windowed grouped-query attention (norms over the whole q and k projections, no rotation, a
learned bias by head and bucket of distance, one added to the softmax's denominator) or latent attention over every key:
with queries straight from the stream, a rotation of split halves with frequencies stretched by pair index and an output
gate per element, or with queries through a latent, a rotation of adjacent pairs and an output gate per head.  The
feed-forward squares a relu.  An entry of the layer list may run another entry's weights again (with a cache of its own).
The embedding is multiplied by a constant; the head has a matrix of its own.  Tensor names are the checkpoint's:
`l<i>.norm1`, `l<i>.mix.rel`, `l<i>.mix.dkv`, `l<i>.mlp.up`, `embed`, `final.norm`, `head`.
"""
from __future__ import annotations

from ..config.zazerax import ZazeraxConfig
from ..parts.base import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

BIAS_ROWS = 32              # rows of the distance biases where neither a checkpoint nor the configuration says
SINK = 0.0                  # the sink's score: one is added to the softmax's denominator
ATTENTION_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.", "k_norm": "k.", "distance": "rel"}


def _norm(width: int, eps: float, name: str) -> PartSpec:
    return PartSpec("layernorm", {"size": width, "eps": eps, "name": name, "bias_name": None})


def _mixer(kind: str, m, W: int, eps: float, bias_rows: int) -> PartSpec:
    if kind == "attention":
        return PartSpec("paged_attention", {
            "hidden_size": W, "n_heads": m.heads, "n_kv_heads": m.kv_heads, "head_dim": m.dim, "v_dim": m.vdim, "bias": False,
            "scale": m.scale, "window": m.window, "position": PartSpec("none", {"head_dim": m.dim}),
            "qk_norm": PartSpec("rmsnorm", {"size": m.dim, "eps": eps, "name": "norm"}), "qk_norm_span": "projection",
            "distance_buckets": (bias_rows, m.bias_max), "sink_value": SINK, "names": ATTENTION_NAMES,
        }, prefix="mix.")
    position = PartSpec("none", {"head_dim": m.rot_dim})
    if m.rot is not None:
        position = PartSpec("rope_ramped", {"head_dim": m.rot_dim, "theta": m.rot.base, "rotary_dim": m.rot.dims,
                                            "interleaved": kind == "latent_attention_2", "scaling": m.rot.scaling})
    return PartSpec("latent_attention", {
        "hidden_size": W, "n_heads": m.heads, "head_dim": m.dim, "rot_dim": m.rot_dim, "v_dim": m.vdim, "q_rank": m.q_rank,
        "kv_rank": m.kv_rank, "scale": m.scale, "latent_norm": PartSpec("rmsnorm", {"eps": eps, "name": "norm"}),
        "position": position, "out_gate": "head" if kind == "latent_attention_2" else "element",
    }, prefix="mix.")


def build_spec(cfg: ZazeraxConfig, tensor_names=None) -> ModelSpec:
    W, eps = cfg.width, cfg.eps
    shapes = getattr(tensor_names, "shapes", {})
    layers, place = [], {}         # place: entry -> index into `layers` of the one whose tensors it runs
    for i, layer in enumerate(cfg.layers):
        if layer.weights_of is not None:
            continue
        m = layer.mixer
        shape = shapes.get(f"l{i}.mix.rel")      # the table's size is the checkpoint's
        rows = int(shape[0]) if shape else (getattr(m, "bias_rows", None) or BIAS_ROWS)
        parts = {"norm1": _norm(W, eps, "norm1"), "mixer": _mixer(layer.type, m, W, eps, rows)}
        if layer.mlp is not None:
            parts["norm2"] = _norm(W, eps, "norm2")
            parts["ffn"] = PartSpec("mlp", {"hidden_size": W, "intermediate_size": layer.mlp.ff, "activation": "relu2",
                                            "names": {"up": "up", "down": "down"}}, prefix="mlp.")
        place[i] = len(layers)
        layers.append(LayerSpec("postnorm", f"l{i}.", parts))
    return ModelSpec(
        hidden_size=W, vocab_size=cfg.vocab,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": W, "name": "embed",
                                               "scale": cfg.embedding_scale}),
        layers=layers,
        schedule=[ScheduleEntry(place[i if layer.weights_of is None else layer.weights_of]) for i, layer in enumerate(cfg.layers)],
        final_norm=_norm(W, eps, "final.norm"),
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "hidden_size": W, "name": "head"}),
        max_positions=cfg.max_positions,
        eos_token_id=cfg.eos_token_id,
    )
