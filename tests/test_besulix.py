"""Besulix on the CPU: the plain model's own properties (it is the judge of the GPU tests), the configuration reader
and its refusals, and the tensor names and shapes of the model description against a list written from the design."""
import copy
import math

import pytest
import torch

import besulix_util as u
import plain_besulix as plain

F64 = torch.float64


def rand(*shape, seed=0):
    return torch.randn(*shape, dtype=F64, generator=torch.Generator().manual_seed(seed))


# ---------------------------------------------------------------------------
# the plain model
# ---------------------------------------------------------------------------
def test_rotation_depends_on_the_distance_alone():
    q, k = rand(1, 1, 12), rand(1, 1, 12, seed=1)

    def score(i, j):
        return float((plain.turn(q, torch.tensor([i]), 50.0) * plain.turn(k, torch.tensor([j]), 50.0)).sum())
    assert score(9, 4) == pytest.approx(score(25, 20)) and abs(score(9, 4) - score(9, 5)) > 1e-3


def test_only_the_first_dimensions_of_a_head_are_rotated_in_halves():
    x = rand(5, 2, 10)
    y = plain.rotary(x, torch.arange(5), 100.0, 6)
    assert torch.equal(y[..., 6:], x[..., 6:]) and torch.allclose(y[0], x[0])
    a = 3 * 100.0 ** (-2 / 6)                     # pair 1 of three at position 3: elements 1 and 4
    assert float(y[3, 0, 1]) == pytest.approx(float(x[3, 0, 1] * math.cos(a) - x[3, 0, 4] * math.sin(a)))
    assert float(y[3, 0, 4]) == pytest.approx(float(x[3, 0, 4] * math.cos(a) + x[3, 0, 1] * math.sin(a)))


def test_a_value_turned_and_turned_back_at_its_own_position_is_itself():
    v, pos = rand(7, 2, 8), torch.arange(7) * 13
    assert torch.allclose(plain.turn(plain.turn(v, pos, 77.0), pos, 77.0, sign=-1.0), v)


def test_chunks_count_from_the_sequences_start():
    vis = plain.chunk_visible(12, 5)
    assert vis[4].tolist() == [True] * 5 + [False] * 7
    assert vis[5].tolist() == [False] * 5 + [True] + [False] * 6
    assert vis[11].tolist() == [False] * 10 + [True, True]


def test_a_sink_takes_weight_and_gives_nothing():
    s, vis = rand(3, 4), torch.ones(3, 4, dtype=torch.bool)
    w = plain.softmax_with_sink(s, vis, torch.tensor(0.5, dtype=F64))
    e = torch.exp(s)
    assert torch.allclose(w, e / (e.sum(-1, keepdim=True) + math.exp(0.5)))
    assert torch.all(torch.isfinite(plain.softmax_with_sink(s, vis, torch.tensor(500.0, dtype=F64))))


def test_the_temperature_does_not_touch_the_sink():
    cfg = u.config([u.parallel_layer(heads=1, kv_heads=1)])
    w = u.as_float64(u.make_weights(cfg, 1))
    p, m = "l0.mix.left.", cfg["layers"][0]["mixer"]["left"]
    h = rand(1, cfg["width"])                      # one token: one key, weight e^s / (e^s + e^sink)
    q = (h @ w[p + "q"].T + w[p + "q.b"]).view(-1)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).view(-1)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).view(-1)
    s = float(q @ k) * m["scale"] * float(w[p + "temp"])
    weight = math.exp(s) / (math.exp(s) + math.exp(float(w[p + "sink"])))
    assert torch.allclose(plain.chunked_attention(h, w, p, m)[0], weight * v @ w[p + "o"].T)


def test_time_mixing_reads_the_state_before_the_token_and_the_bonus_for_it():
    """One head of two channels, by hand."""
    W, D = 4, 2
    g = torch.Generator().manual_seed(3)
    w = {s: torch.randn(D, W, generator=g, dtype=F64) for s in "rkvg"}
    w.update({f"mu.{s}": torch.rand(W, generator=g, dtype=F64) for s in "rkvgw"})
    w.update({"w1": torch.randn(3, W, generator=g, dtype=F64), "w2": torch.randn(D, 3, generator=g, dtype=F64),
              "w0": torch.randn(D, generator=g, dtype=F64), "u": torch.randn(1, D, generator=g, dtype=F64),
              "norm": torch.ones(D, dtype=F64), "o": torch.randn(W, D, generator=g, dtype=F64)})
    h = rand(2, W, seed=9)
    y = plain.time_mix(h, w, "", {"heads": 1, "dim": D}, 0.0)

    def mix(t, s):
        before = h[t - 1] if t else torch.zeros(W, dtype=F64)
        return h[t] + (before - h[t]) * w["mu." + s]
    r, k, v = ([w[s] @ mix(t, s) for t in (0, 1)] for s in "rkv")
    o0 = (r[0] * w["u"][0] * k[0]).sum() * v[0]
    o1 = (r[1] * k[0]).sum() * v[0] + (r[1] * w["u"][0] * k[1]).sum() * v[1]      # (no decay between two neighbours)
    for t, o in ((0, o0), (1, o1)):
        gate = w["g"] @ mix(t, "g")
        want = w["o"] @ (o / torch.sqrt((o * o).mean()) * gate / (1 + torch.exp(-gate)))
        assert torch.allclose(y[t], want)
    d = plain.channel_decay(torch.stack([mix(1, "w")]), w, "")
    assert torch.allclose(d[0], torch.exp(-torch.exp(w["w0"] + w["w2"] @ torch.tanh(w["w1"] @ mix(1, "w")))))
    assert float(d.max()) < 1.0 and float(d.min()) > 0.0


def test_matrix_memory_starts_its_maximum_at_zero():
    cfg = u.config([u.mlstm_layer()])
    w = u.as_float64(u.make_weights(cfg, 1))
    m, h = cfg["layers"][0]["mixer"], rand(1, cfg["width"])
    outs = []
    for bias in (-5.0, -6.0):         # i far below 0: m stays 0, the write is exp(i)
        w["l0.mix.i.b"] = torch.full_like(w["l0.mix.i.b"], bias)
        outs.append(plain.matrix_memory(h, w, "l0.mix.", m, 1e-6))
    assert not torch.allclose(outs[0], outs[1], rtol=1e-3), "a maximum that started at minus infinity would hide the input gate"


def test_the_feed_forward_clamps_the_gate_from_above_and_up_on_both_sides():
    w = {"gate": torch.eye(3, dtype=F64), "up": torch.eye(3, dtype=F64), "down": torch.eye(3, dtype=F64)}
    y = plain.clamped_ff(torch.tensor([[9.0, -9.0, 0.25]], dtype=F64), w, "", 0.5)[0]

    def unit(g, up):
        return g / (1 + math.exp(-1.702 * g)) * (up + 1)
    assert [float(v) for v in y] == pytest.approx([unit(0.5, 0.5), unit(-9.0, -0.5), unit(0.25, 0.25)])


def test_logits_are_capped():
    z = torch.tensor([-1e6, 0.0, 1.0, 1e6], dtype=F64)
    assert torch.allclose(plain.capped(z, 7.0), torch.tensor([-7.0, 0.0, 7.0 * math.tanh(1 / 7), 7.0], dtype=F64))


def test_the_plain_model_is_causal_and_depends_on_every_tensor():
    cfg = u.CFG_MAIN
    w = u.as_float64(u.make_weights(cfg, 3))
    tokens = u.random_tokens(cfg["vocab"], 30, 1)
    base = plain.forward(cfg, w, tokens)
    assert torch.allclose(plain.forward(cfg, w, tokens[:17]), base[:17], atol=1e-9)
    spread = float(base.std())
    for name in w:
        w2 = dict(w)
        w2[name] = w[name] * 1.5 + torch.linspace(0.0, 0.5, w[name].numel(), dtype=F64).view_as(w[name])     # (no uniform shift or factor)
        assert float((plain.forward(cfg, w2, tokens) - base).abs().max()) > 1e-3 * spread, name


def test_the_plain_model_moves_when_a_constant_of_the_configuration_does():
    cfg = u.CFG_MAIN
    w = u.as_float64(u.make_weights(cfg, 3))
    tokens = u.random_tokens(cfg["vocab"], 60, 5)
    base = plain.forward(cfg, w, tokens)

    def moved(other):
        return float(u.row_errors(plain.forward(other, w, tokens), base).max())
    for layer, key, value in ((1, "left__scale", 0.5), (1, "left__mask", {"size": 25}), (1, "left__rot", {"base": 9000.0, "dims": 8}),
                              (1, "left__rot", {"base": 10000.0, "dims": 10}), (1, "left_scale", 0.8), (2, "right_scale", 0.8),
                              (0, "gate_cap", 1.0), (4, "left__mask", {"size": 49})):
        assert moved(u.changed(cfg, layer, **{key: value})) > 5 * u.EDGE_LIMIT["float32"], (layer, key)
    assert moved({**cfg, "logit_softcap": 50.0}) > u.EDGE_LIMIT["bfloat16"]
    assert moved({**cfg, "norm": {"eps": 1e-2}}) > 5 * u.EDGE_LIMIT["float32"]
    free = copy.deepcopy(cfg)
    free["layers"][1]["mlp"]["limit"] = 100.0
    assert moved(free) > u.EDGE_LIMIT["bfloat16"] / 2


# ---------------------------------------------------------------------------
# configuration and description
# ---------------------------------------------------------------------------
def test_configuration_reads_every_size_and_constant():
    from ferrox_amd.config.besulix import BesulixConfig
    cfg = BesulixConfig.from_dict(copy.deepcopy(u.CFG_MAIN))
    assert (cfg.vocab, cfg.width, cfg.eps, cfg.logit_softcap) == (150, 48, 1e-5, 5.0)
    assert [layer.type for layer in cfg.layers] == ["mlstm", "parallel", "parallel", "mlstm", "parallel"]
    m = cfg.layers[2].mixer
    assert (m.left.heads, m.left.kv_heads, m.left.dim, m.left.vdim, m.left.scale) == (3, 3, 12, 20, 0.45)
    assert (m.left.rot_dims, m.left.rot_base, m.left.chunk) == (12, 500.0, 7)
    assert (m.right.heads, m.right.dim, m.left_scale, m.right_scale) == (2, 20, 1.0, -0.8)
    n = cfg.layers[3].mixer
    assert (n.heads, n.dim, n.vdim, n.gate_cap) == (2, 20, 8, 4.0) and cfg.layers[3].mlp is None
    assert (cfg.layers[4].mlp.ff, cfg.layers[4].mlp.limit) == (56, 3.0)
    assert cfg.to_dict()["layers"] == u.CFG_MAIN["layers"]


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0].update(type="attention"), "type 'attention'"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=3), "multiple of kv_heads"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(vdim=11), "even"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(dim=300), "attention kernels"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=7), "even and at most"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=18), "even and at most"),
    (lambda c: c["layers"][1]["mixer"]["left"].pop("mask"), "mask"),
    (lambda c: c["layers"][1]["mixer"].pop("right_scale"), "right_scale"),
    (lambda c: c["layers"][2]["mixer"]["right"].update(dim=257), "256 key channels"),
    (lambda c: c["layers"][3]["mixer"].update(gate_cap=0.0), "gate_cap"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "kind 'moe'"),
    (lambda c: c["layers"][0]["mlp"].pop("limit"), "limit"),
    (lambda c: c.pop("logit_softcap"), "logit_softcap"),
    (lambda c: c.update(layers=[]), "layers"),
])
def test_configuration_refuses(change, message):
    from ferrox_amd.config.base import ConfigError
    from ferrox_amd.config.besulix import BesulixConfig
    raw = copy.deepcopy(u.CFG_MAIN)
    change(raw)
    with pytest.raises(ConfigError, match=message):
        BesulixConfig.from_dict(raw)


@pytest.mark.parametrize("cfg, rank", [(u.CFG_MAIN, 5), (u.CFG_MFMA, 24), (u.config([u.mlstm_layer()]), 5)])
def test_description_names_the_designs_tensors(cfg, rank):
    from ferrox_amd.engine.model import Model
    from ferrox_amd.models.registry import resolve
    arch = resolve(cfg)
    assert arch.name == "Besulix"
    shapes = u.tensor_shapes(cfg, rank)

    class Names(list):          # what the loader hands over: the checkpoint's names with their shapes
        pass
    names = Names(shapes)
    names.shapes = shapes
    model = Model(arch.build_spec(arch.config_class.from_dict(copy.deepcopy(cfg)), names))
    assert {name: tuple(spec.shape) for name, spec in model.named_params().items()} == shapes
    assert all(b.mixer.graph_safe for b in model.blocks), "decode steps of this design are recorded"
    chunks = {layer["mixer"]["left"]["mask"]["size"] for layer in cfg["layers"] if layer["type"] == "parallel"}
    assert model.cache_groups() == {("chunk", c): ("chunk", c) for c in chunks}


def test_without_a_checkpoint_the_decays_inner_size_is_the_configurations():
    from ferrox_amd.engine.model import Model
    from ferrox_amd.models.registry import resolve
    cfg = u.changed(u.CFG_MAIN, 1, right__decay_rank=9)
    arch = resolve(cfg)
    params = Model(arch.build_spec(arch.config_class.from_dict(cfg), None)).named_params()
    assert tuple(params["l1.mix.right.w1"].shape) == (9, 48) and tuple(params["l2.mix.right.w2"].shape) == (40, 16)


def test_the_values_channels_are_reordered_into_neighbouring_pairs():
    from ferrox_amd.parts.attention import PagedAttention
    from ferrox_amd.parts.base import PartSpec
    common = dict(hidden_size=8, n_heads=2, n_kv_heads=1, head_dim=4, v_dim=6, bias=True, value_rotation=100.0)
    halves = PagedAttention(position=PartSpec("rope_neox", {"head_dim": 4, "theta": 100.0}), **common)
    assert halves.value_pair_order().tolist() == [0, 3, 1, 4, 2, 5]
    pairs = PagedAttention(position=PartSpec("rope_interleaved", {"head_dim": 4, "theta": 100.0}), **common)
    assert pairs.value_pair_order().tolist() == list(range(6))
    with pytest.raises(ValueError, match="even"):
        PagedAttention(position=PartSpec("rope_neox", {"head_dim": 4, "theta": 100.0}), **{**common, "v_dim": 5})
    with pytest.raises(ValueError, match="plain projections"):
        PagedAttention(position=PartSpec("rope_neox", {"head_dim": 4, "theta": 100.0}), **{**common, "bias": False}, out_gate=True)


def test_the_named_shape_is_a_configuration_of_the_design():
    from ferrox_amd.config import presets
    from ferrox_amd.config.besulix import BesulixConfig
    cfg = BesulixConfig.from_dict(presets.load("besulix-2k"))
    assert {layer.type for layer in cfg.layers} == {"parallel", "mlstm"} and cfg.width == 2048
