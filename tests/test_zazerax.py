"""Zazerax on the CPU: the plain model's own properties (it is the judge of the GPU tests), the configuration reader and
its refusals, the tensor names and shapes of the model description against a list written from the design, the rows of
the distance biases and the order of rotated pairs that the weights are brought into."""
import bisect
import copy
import math

import pytest
import torch

import plain_zazerax as plain
import zazerax_util as u

F64 = torch.float64


def rand(*shape, seed=0):
    return torch.randn(*shape, dtype=F64, generator=torch.Generator().manual_seed(seed))


# ---------------------------------------------------------------------------
# the plain model
# ---------------------------------------------------------------------------
def test_a_window_holds_the_query_and_the_keys_before_it():
    see = plain.visible(8, 3)
    assert see[7].tolist() == [False] * 5 + [True] * 3
    assert see[1].tolist() == [True, True] + [False] * 6
    assert plain.visible(5).tolist() == torch.tril(torch.ones(5, 5)).bool().tolist()


def test_one_in_the_denominator_takes_weight_and_gives_nothing():
    s = rand(3, 5)
    w = plain.softmax_plus_one(s)
    assert torch.allclose(w, torch.exp(s) / (1 + torch.exp(s).sum(-1, keepdim=True)))
    for far in (-800.0, 800.0):
        assert torch.all(torch.isfinite(plain.softmax_plus_one(s + far)))
    masked = s.masked_fill(torch.tensor([True, False, False, True, False]), -math.inf)
    assert torch.allclose(plain.softmax_plus_one(masked).sum(-1), 1 - 1 / (1 + torch.exp(masked).sum(-1)))


def test_buckets_are_distances_then_widen():
    rows, far = 8, 64                                        # rows 4 .. 7 begin at 4, 8, 16, 32
    assert [plain.bucket(d, rows, far) for d in (0, 3, 4, 7, 8, 15, 16, 31, 32, 63, 64, 10 ** 6)] == [0, 3, 4, 4, 5, 5, 6, 6, 7, 7, 7, 7]
    for rows, far in ((12, 20), (10, 160), (6, 31), (2, 5), (16, 100)):      # the formula with logarithms, where it is not on an edge
        half = rows // 2
        for d in range(half, far + 20):
            x = math.log(d / half) / math.log(far / half) * (rows - half)
            if abs(x - round(x)) > 1e-9:
                assert plain.bucket(d, rows, far) == min(rows - 1, half + math.floor(x)), (rows, far, d)


def test_rotation_depends_on_the_distance_alone_and_pairs_as_told():
    freqs, mag = plain.rotation({"dims": 6, "base": 50.0})
    assert mag == 1.0 and freqs[1] == pytest.approx(50.0 ** (-2 / 6))
    for halves in (True, False):
        q, k = rand(1, 6).expand(12, 6), rand(1, 6, seed=1).expand(12, 6)
        a, b = (plain.rotate(x, freqs, mag, halves, angles="exact") for x in (q, k))
        assert float(a[9] @ b[4]) == pytest.approx(float(a[11] @ b[6])) and abs(float(a[9] @ b[4]) - float(a[9] @ b[5])) > 1e-4
        x = rand(4, 8, seed=2)
        y = plain.rotate(x, freqs, mag, halves, angles="exact")
        assert torch.equal(y[:, 6:], x[:, 6:]) and torch.allclose(y[0], x[0])
        i, j = (1, 4) if halves else (2, 3)                  # pair 1 of three
        t = 3 * freqs[1]
        assert float(y[3, i]) == pytest.approx(float(x[3, i] * math.cos(t) - x[3, j] * math.sin(t)))
        assert float(y[3, j]) == pytest.approx(float(x[3, j] * math.cos(t) + x[3, i] * math.sin(t)))


def test_stretched_frequencies_have_three_bands_and_a_magnitude():
    sc = dict(zip(("factor", "original", "fast", "slow"), (4.0, 40, 4.0, 0.5)))
    f, mag = plain.rotation({"dims": 16, "base": 100.0, "scaling": sc})
    g, _ = plain.rotation({"dims": 16, "base": 100.0})
    ratios = [a / b for a, b in zip(f, g)]
    assert mag == pytest.approx(0.1 * math.log(4.0) + 1.0)
    assert ratios[0] == 1.0 and ratios[-1] == pytest.approx(0.25) and any(0.25 < r < 1.0 for r in ratios) and ratios == sorted(ratios, reverse=True)


def test_the_first_token_alone_by_hand():
    """One key: weight e^s / (1 + e^s) under the biased attention, all of it under latent attention."""
    cfg = u.config([u.attention_layer(heads=1, kv_heads=1, dim=4, vdim=4)], width=8)
    w = u.as_float64(u.make_weights(cfg, 1))
    h, m = rand(1, 8), cfg["layers"][0]["mixer"]
    wm = plain.sub(w, "l0.mix.")
    q, k = plain.rms_norm(h @ wm["q"].T, wm["q.norm"], 1e-6), plain.rms_norm(h @ wm["k"].T, wm["k.norm"], 1e-6)
    s = float(q[0] @ k[0]) * m["scale"] + float(wm["rel"][0, 0])
    want = math.exp(s) / (1 + math.exp(s)) * (h @ wm["v"].T) @ wm["o"].T
    assert torch.allclose(plain.biased_attention(h, wm, m, 1e-6), want)
    for layer, gate in ((u.latent_layer(heads=2), "element"), (u.latent_layer_2(heads=2), "head")):
        cfg = u.config([layer], width=8)
        wm, m = plain.sub(u.as_float64(u.make_weights(cfg, 2)), "l0.mix."), layer["mixer"]
        c = plain.rms_norm((h @ wm["dkv"].T)[:, :m["kv_rank"]], wm["dkv.norm"], 1e-6)
        g = torch.sigmoid(h @ wm["g"].T)
        g = g.repeat_interleave(m["vdim"], dim=1) if gate == "head" else g
        got = plain.latent_attention(h, wm, m, 1e-6, gate == "element", gate)
        assert torch.allclose(got, (c @ wm["uv"].T * g) @ wm["o"].T)


def test_norms_stand_behind_the_sublayers():
    cfg = u.config([u.attention_layer(mlp=u.dense(24))], emb_scale=2.0)
    w = u.as_float64(u.make_weights(cfg, 4))
    tokens, seen = [5, 9, 5], []
    plain.forward(cfg, w, tokens, layers_out=seen)
    x = w["embed"][torch.tensor(tokens)] * 2.0
    mixed = plain.biased_attention(x, plain.sub(w, "l0.mix."), cfg["layers"][0]["mixer"], 1e-6)
    x = x + plain.layer_norm(mixed, w["l0.norm1"], 1e-6)
    up = torch.clamp(x @ w["l0.mlp.up"].T, min=0) ** 2
    assert torch.allclose(seen[0], x + plain.layer_norm(up @ w["l0.mlp.down"].T, w["l0.norm2"], 1e-6))
    y = plain.layer_norm(rand(2, 50) + 3.0, torch.ones(50, dtype=F64), 0.0)
    assert torch.allclose(y.mean(-1), torch.zeros(2, dtype=F64), atol=1e-12) and torch.allclose(y.pow(2).mean(-1), torch.ones(2, dtype=F64))


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
    sc = dict(zip(("factor", "original", "fast", "slow"), u.STRETCH))
    for layer, change in ((0, {"scale": 0.3}), (0, {"mask": {"size": 14}}), (0, {"bias_max": 16}), (3, {"mask": {"size": 29}}),
                          (3, {"bias_max": 18}), (1, {"scale": 0.3}), (1, {"rot": {"base": 100.0, "dims": 8}}),
                          (1, {"rot": {"base": 90.0, "dims": 8, "scaling": sc}}), (1, {"rot": {"base": 100.0, "dims": 8, "scaling": {**sc, "factor": 2.5}}}),
                          (1, {"rot": {"base": 100.0, "dims": 8, "scaling": {**sc, "original": 90}}}), (2, {"rot": {"base": 60.0, "dims": 8}}),
                          (2, {"rot": {"base": 50.0, "dims": 12}}), (6, {"rot": {"base": 200.0, "dims": 12}})):
        assert moved(u.changed(cfg, layer, **change)) > 5 * u.EDGE_LIMIT["float32"], (layer, change)
    assert moved({**cfg, "norm": {"eps": 1e-2}}) > 5 * u.EDGE_LIMIT["float32"]
    assert moved({**cfg, "embedding": {"scale": 1.0}}) > 5 * u.EDGE_LIMIT["float32"]


# ---------------------------------------------------------------------------
# configuration and description
# ---------------------------------------------------------------------------
def read(raw):
    from ferrox_amd.config.zazerax import ZazeraxConfig
    return ZazeraxConfig.from_dict(copy.deepcopy(raw))


def test_configuration_reads_every_size_and_constant():
    cfg = read(u.CFG_MAIN)
    assert (cfg.vocab, cfg.width, cfg.eps, cfg.embedding_scale) == (160, 64, 1e-6, 1.7)
    assert [layer.type for layer in cfg.layers] == [layer["type"] for layer in u.CFG_MAIN["layers"]]
    m = cfg.layers[3].mixer
    assert (m.heads, m.kv_heads, m.dim, m.vdim, m.scale, m.bias_max, m.window) == (3, 3, 24, 16, 0.3, 14, 30)
    m = cfg.layers[1].mixer
    assert (m.heads, m.dim, m.rot_dim, m.vdim, m.q_rank, m.kv_rank, m.scale) == (3, 16, 8, 24, None, 24, 0.35)
    assert (m.rot.dims, m.rot.base, m.rot.scaling) == (8, 100.0, (3.0, 40.0, 4.0, 0.5))
    m = cfg.layers[2].mixer
    assert (m.q_rank, m.rot_dim, m.rot.dims, m.rot.base, m.rot.scaling) == (28, 12, 8, 50.0, None)
    assert cfg.layers[2].mlp is None and cfg.layers[6].mlp.ff == 16
    assert [layer.weights_of for layer in cfg.layers] == [None, None, None, None, 1, 0, None, None]
    assert cfg.to_dict()["layers"] == u.CFG_MAIN["layers"]
    assert read({k: v for k, v in u.CFG_MAIN.items() if k != "embedding"}).embedding_scale == 1.0


def test_weights_may_be_those_of_a_later_layer_or_of_one_that_uses_anothers():
    layers = u._main_layers()
    raw = u.config([u.again(layers, 1), layers[1], {**copy.deepcopy(layers[1]), "weights_of": 0}])
    raw["layers"][0]["weights_of"] = 1
    assert [layer.weights_of for layer in read(raw).layers] == [1, None, 1]
    from ferrox_amd.models.zazerax import build_spec
    spec = build_spec(read(raw))
    assert [layer.prefix for layer in spec.layers] == ["l1."] and [e.layer for e in spec.schedule] == [0, 0, 0]
    assert all(e.cache is None for e in spec.schedule), "every entry has a cache of its own"


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0].update(type="mlstm"), "type 'mlstm'"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "multiple of kv_heads"),
    (lambda c: c["layers"][0]["mixer"].update(dim=300), "attention kernels"),
    (lambda c: c["layers"][0]["mixer"].pop("bias_max"), "bias_max"),
    (lambda c: c["layers"][0]["mixer"].update(scale=0.0), "scale"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=7), "even and at most"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=10), "even and at most"),
    (lambda c: c["layers"][1]["mixer"].update(kv_rank=505), "attention kernels"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(base=1.0), "wavelengths"),
    (lambda c: c["layers"][2]["mixer"].pop("q_rank"), "q_rank"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "kind 'moe'"),
    (lambda c: c["layers"][4].update(weights_of=8), "weights_of names no layer"),
    (lambda c: c["layers"][4].update(weights_of=4), "weights_of names no layer"),
    (lambda c: c["layers"][4].update(weights_of=2), "is not like it"),
    (lambda c: c.pop("norm"), "norm"),
    (lambda c: c.update(layers=[]), "layers"),
])
def test_configuration_refuses(change, message):
    from ferrox_amd.config.base import ConfigError
    raw = copy.deepcopy(u.CFG_MAIN)
    change(raw)
    with pytest.raises(ConfigError, match=message):
        read(raw)


@pytest.mark.parametrize("cfg, rows", [(u.CFG_MAIN, 12), (u.CFG_MFMA, 16), (u.config([u.attention_layer()], emb_scale=None), 4)])
def test_description_names_the_designs_tensors(cfg, rows):
    from ferrox_amd.engine.model import Model
    from ferrox_amd.models.registry import resolve
    arch = resolve(cfg)
    assert arch.name == "Zazerax"
    shapes = u.tensor_shapes(cfg, rows)

    class Names(list):          # what the loader hands over: the checkpoint's names with their shapes
        pass
    names = Names(shapes)
    names.shapes = shapes
    model = Model(arch.build_spec(read(cfg), names))
    assert {name: tuple(spec.shape) for name, spec in model.named_params().items()} == shapes
    assert all(b.mixer.graph_safe for b in model.blocks), "decode steps of this design are recorded"
    groups = {("window", layer["mixer"]["mask"]["size"]): layer["mixer"]["mask"]["size"] for layer in cfg["layers"] if layer["type"] == "attention"}
    if any(layer["type"] != "attention" for layer in cfg["layers"]):
        groups[("full",)] = None
    assert model.cache_groups() == groups


def test_without_a_checkpoint_the_biases_rows_are_the_configurations():
    from ferrox_amd.engine.model import Model
    from ferrox_amd.models.zazerax import BIAS_ROWS, build_spec
    raw = u.config([u.attention_layer(bias_max=99), u.attention_layer(bias_max=99)])
    raw["layers"][1]["mixer"]["bias_rows"] = 9
    params = Model(build_spec(read(raw))).named_params()
    assert tuple(params["l0.mix.rel"].shape) == (BIAS_ROWS, 4) and tuple(params["l1.mix.rel"].shape) == (9, 4)


def test_rows_of_the_distance_biases():
    from ferrox_amd.parts.attention import PagedAttention, bucket_starts
    from ferrox_amd.parts.base import PartSpec
    for rows, far in ((12, 20), (10, 160), (8, 64), (8, 100), (32, 128), (2, 5), (3, 9), (6, 31), (16, 17)):
        starts = bucket_starts(rows, far)
        assert len(starts) == rows and starts == sorted(starts)
        assert [bisect.bisect_right(starts, d) - 1 for d in range(far + 40)] == [plain.bucket(d, rows, far) for d in range(far + 40)], (rows, far)

    def part(window, buckets, **kw):
        return PagedAttention(hidden_size=8, n_heads=2, n_kv_heads=1, head_dim=4, bias=False, window=window, distance_buckets=buckets,
                              position=PartSpec("none", {"head_dim": 4}), **kw)
    assert part(7, (8, 64)).distance_rows() == [0, 1, 2, 3, 4, 4, 4]                     # no farther than a window sees
    assert part(None, (8, 64)).distance_rows() == [plain.bucket(d, 8, 64) for d in range(33)]      # nor than the last row's start
    assert part(3, (8, 3)).distance_rows() == [0, 1, 2]                                  # a window within the rows that hold one distance each
    with pytest.raises(ValueError, match="last row"):
        part(30, (8, 4))
    with pytest.raises(ValueError, match="learned or one"):
        part(7, (8, 64), sink=True, sink_value=0.0)


def test_the_bias_table_runs_from_far_to_near():
    from ferrox_amd import ops
    t = ops.distance_bias_rows(torch.tensor([[1.0, 2.0, 3.0], [4.0, 5.0, 6.0]]))
    pad = ops.BIAS_PAD
    assert t.shape == (2, 3 + 2 * pad) and t[1, pad:pad + 3].tolist() == [6.0, 5.0, 4.0]
    assert t[0, :pad].tolist() == [3.0] * pad and t[0, pad + 3:].tolist() == [0.0] * pad


def test_rotated_halves_become_neighbours():
    from ferrox_amd.parts.base import PartSpec
    from ferrox_amd.parts.latent import LatentAttention

    def part(interleaved, dims, **kw):
        args = dict(hidden_size=8, n_heads=2, head_dim=4, rot_dim=8, v_dim=6, q_rank=None, kv_rank=4, scale=0.5,
                    latent_norm=PartSpec("rmsnorm", {"eps": 1e-5, "name": "norm"}),
                    position=PartSpec("rope_ramped", {"head_dim": 8, "theta": 100.0, "rotary_dim": dims, "interleaved": interleaved}))
        return LatentAttention(**{**args, **kw})
    assert part(False, 6).pair_order().tolist() == [0, 3, 1, 4, 2, 5, 6, 7]
    assert part(True, 6).pair_order().tolist() == list(range(8))
    assert part(False, 0).pair_order().tolist() == list(range(8))
    with pytest.raises(ValueError, match="out_gate"):
        part(True, 8, out_gate="row")
    with pytest.raises(ValueError, match="keys of their own"):
        part(True, 8, own_kv=False)


def test_a_post_norm_block_has_both_halves_of_a_feed_forward_or_none():
    from ferrox_amd.engine.model import Model
    from ferrox_amd.models.zazerax import build_spec
    spec = build_spec(read(u.CFG_MAIN))
    del spec.layers[0].parts["norm2"]
    with pytest.raises(ValueError, match="or neither"):
        Model(spec)


def test_the_named_shape_is_a_configuration_of_the_design():
    from ferrox_amd.config import presets
    from ferrox_amd.config.zazerax import MIXER_TYPES
    cfg = read(presets.load("zazerax-2k"))
    assert {layer.type for layer in cfg.layers} == set(MIXER_TYPES) and cfg.width == 2048
    assert any(layer.weights_of is not None for layer in cfg.layers)
