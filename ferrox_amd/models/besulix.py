"""Besulix as a list of parts.

Every layer is a pre-norm block, x += mixer(N1(x)), x += ff(N2(x)), N an RMS norm; a layer may have no feed-forward.  The
mixer is a matrix memory with exponential gates, or two mixers side by side, weighted by constants: softmax attention
inside chunks of positions (biases, keys and queries rotated in halves, values rotated by position and turned back at
the query, a temperature and a sink per head) and a time-mixing recurrence with a decay per token and key channel.  The
feed-forward clamps gate and up.  The embedded token is normed before the first layer; the logits are capped.  Tensor
names are the checkpoint's: `l<i>.norm1`, `l<i>.mix.q`, `l<i>.mix.left.q.b`, `l<i>.mix.right.mu.r`, `l<i>.mlp.gate`, `embed`,
`embed.norm`, `final.norm`, `head`.
"""
from __future__ import annotations

from ..config.besulix import BesulixConfig
from ..parts.base import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

GATE_SLOPE = 1.702          # a feed-forward's gate is g * sigmoid(1.702 g)
ATTENTION_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_bias": "q.b", "k_bias": "k.b", "v_bias": "v.b", "sink": "sink",
                   "temperature": "temp"}


def _norm(width: int, eps: float, name: str) -> PartSpec:
    return PartSpec("rmsnorm", {"size": width, "eps": eps, "name": name})


def _side_by_side(m, W: int, eps: float, decay_rank: int) -> PartSpec:
    left, right = m.left, m.right
    return PartSpec("side_by_side", {
        "members": {
            "left": PartSpec("paged_attention", {
                "hidden_size": W, "n_heads": left.heads, "n_kv_heads": left.kv_heads, "head_dim": left.dim, "v_dim": left.vdim,
                "bias": True, "scale": left.scale, "chunk": left.chunk, "sink": True, "head_temperature": True,
                "value_rotation": left.rot_base,
                "position": PartSpec("rope_neox", {"head_dim": left.dim, "theta": left.rot_base, "rotary_dim": left.rot_dims}),
                "names": ATTENTION_NAMES,
            }, prefix="left."),
            "right": PartSpec("time_mix", {
                "hidden_size": W, "n_heads": right.heads, "head_dim": right.dim, "norm_eps": eps, "decay_rank": decay_rank,
            }, prefix="right."),
        },
        "scales": {"left": m.left_scale, "right": m.right_scale},
    }, prefix="mix.")


def build_spec(cfg: BesulixConfig, tensor_names=None) -> ModelSpec:
    W, eps = cfg.width, cfg.eps
    shapes = getattr(tensor_names, "shapes", {})
    layers = []
    for i, layer in enumerate(cfg.layers):
        m = layer.mixer
        if layer.type == "parallel":
            shape = shapes.get(f"l{i}.mix.right.w1")      # the decay projection's inner size is the checkpoint's
            rank = int(shape[0]) if shape else (m.right.decay_rank or max(16, m.right.dim // 4))
            mixer = _side_by_side(m, W, eps, rank)
        else:
            mixer = PartSpec("matrix_memory", {"hidden_size": W, "n_heads": m.heads, "key_dim": m.dim, "v_dim": m.vdim,
                                               "gate_cap": m.gate_cap, "norm_eps": eps}, prefix="mix.")
        parts = {"norm1": _norm(W, eps, "norm1"), "mixer": mixer}
        if layer.mlp is not None:
            parts["norm2"] = _norm(W, eps, "norm2")
            parts["ffn"] = PartSpec("gated_mlp", {
                "hidden_size": W, "intermediate_size": layer.mlp.ff, "activation": "swiglu_clamped",
                "activation_params": (layer.mlp.limit, GATE_SLOPE), "names": {"gate": "gate", "up": "up", "down": "down"},
            }, prefix="mlp.")
        layers.append(LayerSpec("prenorm", f"l{i}.", parts))
    return ModelSpec(
        hidden_size=W, vocab_size=cfg.vocab,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": W, "name": "embed",
                                               "norm": _norm(W, eps, "embed.norm")}),
        layers=layers,
        schedule=[ScheduleEntry(i) for i in range(len(layers))],
        final_norm=_norm(W, eps, "final.norm"),
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "hidden_size": W, "name": "head", "softcap": cfg.logit_softcap}),
        max_positions=cfg.max_positions,
        eos_token_id=cfg.eos_token_id,
    )
