"""Zazerax on the GPU against the plain model (`plain_zazerax`): every mechanism alone, the new kernels alone, whole
prompts, decoding through the caches, portions down to two tokens, unequal batches, pages and slots used again, keys just
inside and outside windows and at page borders in prompts and in decoding, the first tokens, far keys, long decoding,
other sizes, and generation through the engine's entry points."""
import math

import pytest
import torch

import plain_zazerax as plain
import zazerax_util as u

pytestmark = pytest.mark.gpu

_models = {}
F64 = torch.float64
DTYPES = ["float32", "bfloat16"]


def model_for(tmp_path_factory, name, cfg, seed, dtype, change=None, bias_rows=u.BIAS_ROWS):
    """(weights as the plain model reads them, loaded engine model); made once per (name, dtype)."""
    from ferrox_amd.engine.loading import load_model
    key = (name, dtype)
    if key not in _models:
        weights = u.make_weights(cfg, seed, bias_rows)
        if change:
            change(weights)
        folder = u.write_model(str(tmp_path_factory.mktemp(f"zazerax_{name}")), cfg, weights)
        _models[key] = (weights, load_model(folder, dtype, "cuda:0"))
    return _models[key]


def runner_of(model, block_size=16, num_pages=24, max_seqs=4, **kw):
    from ferrox_amd.engine.runner import ModelRunner
    return ModelRunner(model, block_size=block_size, num_pages=num_pages, max_seqs=max_seqs, **kw)


def run_and_check(cfg, weights, model, requests, schedule, dtype, what, limit=None, **runner_kw):
    runner = runner_of(model, **runner_kw)
    got, _ = u.run_schedule(runner, requests, schedule)
    for key in runner.manager.groups:
        assert runner.manager.n_free_pages(key) == runner_kw.get("num_pages", 24), "pages were lost"
    return u.check_against_plain(cfg, weights, requests, got, dtype, what, limit)


# ---------------------------------------------------------------------------
# each mechanism alone: models of one or two layers
# ---------------------------------------------------------------------------
SINGLE = {
    "attention": u.config([u.attention_layer()]),
    "attention_one_key_head": u.config([u.attention_layer(heads=5, kv_heads=1, dim=8, vdim=24, bias_max=9, window=11)]),
    "attention_biases_end_before_the_window": u.config([u.attention_layer(heads=2, kv_heads=2, bias_max=8, window=40)]),
    "attention_biases_end_behind_the_window": u.config([u.attention_layer(bias_max=300, window=17)]),
    "attention_window_of_one": u.config([u.attention_layer(window=1)]),
    "attention_no_window": u.config([u.attention_layer(window=0, bias_max=26)]),
    "latent": u.config([u.latent_layer()]),
    "latent_plain_frequencies": u.config([u.latent_layer(scaling=None)]),
    "latent_part_turned": u.config([u.latent_layer(heads=1, rot_dim=12, rot_dims=4, kv_rank=20, vdim=8)]),
    "latent_nothing_turned": u.config([u.latent_layer(rot_dim=4, rot_dims=0, scaling=None)]),
    "latent_odd_rotated_part": u.config([u.latent_layer(heads=3, dim=5, rot_dim=7, rot_dims=6, kv_rank=9, vdim=11)]),
    "latent_2": u.config([u.latent_layer_2()]),
    "latent_2_stretched": u.config([u.latent_layer_2(heads=7, dim=12, rot_dim=12, rot_dims=8, q_rank=9, kv_rank=17, vdim=5, scaling=u.STRETCH)]),
    "feed_forward": u.config([u.latent_layer_2(heads=1, mlp=u.dense(56))], eps=1e-3, emb_scale=None),
    "twice": (lambda one: u.config([one, u.again([one], 0), u.again([one], 0)]))(u.attention_layer(mlp=u.dense(24))),
    "twice_latent": (lambda one: u.config([one, u.again([one], 0)]))(u.latent_layer(mlp=u.dense(24))),
}


@pytest.mark.parametrize("name", sorted(SINGLE))
def test_each_mechanism_alone(tmp_path_factory, name):
    cfg = SINGLE[name]
    for dtype in DTYPES:
        weights, model = model_for(tmp_path_factory, name, cfg, 11, dtype)
        reqs = {"a": u.random_tokens(cfg["vocab"], 45, 1), "b": u.random_tokens(cfg["vocab"], 19, 2)}
        run_and_check(cfg, weights, model, reqs, [[("a", 45)], [("b", 19)]], dtype, name + " whole")
        cut = [[("a", 17), ("b", 2)], [("a", 1), ("b", 16)], [("a", 20), ("b", 1)]] + [[("a", 1)]] * 7
        run_and_check(cfg, weights, model, reqs, cut, dtype, name + " cut")


def test_the_comparison_sees_every_mechanism(monkeypatch):
    """The plain model without one mechanism is far beyond the limits of the comparisons in this file."""
    cfg = u.CFG_MAIN
    w = u.as_float64(u.make_weights(cfg, 3))
    tokens = u.random_tokens(cfg["vocab"], 60, 5)
    base = plain.forward(cfg, w, tokens)
    sight = u.EDGE_LIMIT["bfloat16"]

    def moved(other=cfg, **replace):
        return float(u.row_errors(plain.forward(other, dict(w, **replace), tokens), base).max())

    assert moved(**{"l0.mix.rel": torch.zeros_like(w["l0.mix.rel"])}) > sight
    for layer in (1, 2):
        assert moved(**{f"l{layer}.mix.g": torch.zeros_like(w[f"l{layer}.mix.g"])}) > sight / 2
    assert moved(**{"l2.mix.dq.norm": torch.ones_like(w["l2.mix.dq.norm"])}) > 10 * u.EDGE_LIMIT["float32"]
    assert moved(u.changed(cfg, 1, rot={"base": 100.0, "dims": 8})) > 100 * u.EDGE_LIMIT["float32"]
    rotate, softmax, norm, mlp = plain.rotate, plain.softmax_plus_one, plain.layer_norm, plain.squared_relu_mlp
    for name, other in (("softmax_plus_one", lambda s: torch.softmax(s, -1)),
                        ("rotate", lambda v, f, m, halves, a="float32": rotate(v, f, m, not halves, a)),
                        ("layer_norm", lambda x, g, eps: plain.rms_norm(x, g, eps)),
                        ("squared_relu_mlp", lambda h, p: torch.clamp(h @ p["up"].T, min=0.0) @ p["down"].T)):
        monkeypatch.setattr(plain, name, other)
        assert moved() > sight, name
        monkeypatch.undo()
    assert (rotate, softmax, norm, mlp) == (plain.rotate, plain.softmax_plus_one, plain.layer_norm, plain.squared_relu_mlp)


# ---------------------------------------------------------------------------
# the new kernels alone, against torch in float64
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H", [7, 256, 2048, 4096, 4500])
def test_layer_norm_as_rows_join_the_stream(dtype, H):
    from ferrox_amd import ops
    gen = torch.Generator().manual_seed(H)
    h, y = torch.randn(5, H, generator=gen), torch.randn(5, H, generator=gen) * 3 + 2
    w, b = torch.randn(H, generator=gen), torch.randn(H, generator=gen)
    for bias in (None, b):
        want = h.to(F64) + plain.layer_norm(y.to(F64), w.to(F64), 1e-3) + (0 if bias is None else bias.to(F64))
        hd = h.clone().cuda()
        rows = ops.layernorm_add(hd, y.cuda(), w.cuda(), None if bias is None else bias.cuda(), 1e-3, dtype)
        assert torch.allclose(hd.cpu().to(F64), want, rtol=1e-5, atol=1e-5)
        assert rows.dtype == dtype and torch.equal(rows, hd.to(dtype)), "the rows are the stream's, rounded once"
        again = h.clone().cuda()
        assert ops.layernorm_add(again, y.cuda(), w.cuda(), None if bias is None else bias.cuda(), 1e-3) is None
        assert torch.equal(again, hd)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_gated_products_of_every_kind_of_kernel(dtype):
    """The gate in the epilogues of grouped products (a head a group, gate columns beside other columns of wider rows) for
    few rows and many, of sizes that fit no vector, and of a plain product."""
    from ferrox_amd import ops
    from ferrox_amd.parts.latent import head_groups
    gen = torch.Generator().manual_seed(7)
    for T, H, N, K in ((1, 3, 24, 64), (2, 16, 128, 192), (9, 4, 48, 96), (70, 5, 33, 52), (300, 2, 128, 64), (513, 3, 200, 128), (40, 6, 10, 20)):
        a = torch.randn(T * H, K, generator=gen).to(dtype).cuda()
        w = (torch.randn(H, N, K, generator=gen) / K ** 0.5).to(dtype).cuda()
        wide = torch.randn(T, 5 + H * N, generator=gen).cuda() * 2
        gate = wide[:, 5:]
        rows, offsets = head_groups(a.device, T, H)
        out = torch.full((T * H, N), float("nan"), dtype=dtype, device="cuda")
        ops.gemm(a, w, a_rows=rows, c_rows=rows, expert_offsets=offsets, n_rows=T * H, out=out, out_gate=(gate, H))
        z = torch.matmul(a.double().view(T, H, 1, K), w.double().transpose(1, 2).contiguous()).view(T, H * N) * torch.sigmoid(gate.double())
        tol = dict(rtol=1e-4, atol=1e-5) if dtype == torch.float32 else dict(rtol=1e-2, atol=1e-2)
        assert torch.allclose(out.double().view(T, H * N), z, **tol), (T, H, N, K)
    for M, N, K in ((3, 40, 64), (300, 384, 128), (33, 70, 52)):
        a, w = torch.randn(M, K, generator=gen).to(dtype).cuda(), (torch.randn(N, K, generator=gen) / K ** 0.5).to(dtype).cuda()
        gate = torch.randn(M, N, generator=gen).cuda()
        got = ops.gemm(a, w, epilogue=ops.EPI_STORE_F32, out_gate=(gate, 1))
        assert torch.allclose(got.double(), (a.double() @ w.double().t()) * torch.sigmoid(gate.double()), rtol=1e-4, atol=1e-4), (M, N, K)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_squared_relu_of_every_kind_of_kernel(dtype):
    from ferrox_amd import ops
    gen = torch.Generator().manual_seed(8)
    for M, N, K in ((1, 512, 128), (3, 200, 64), (300, 384, 128), (33, 70, 52), (2048, 512, 64), (700, 640, 192)):
        a, w = torch.randn(M, K, generator=gen).to(dtype).cuda(), (torch.randn(N, K, generator=gen) / K ** 0.5).to(dtype).cuda()
        got = ops.gemm(a, w, store_activation="relu2")
        want = torch.clamp(a.double() @ w.double().t(), min=0.0) ** 2
        tol = dict(rtol=1e-4, atol=1e-5) if dtype == torch.float32 else dict(rtol=1e-2, atol=1e-3)
        assert torch.allclose(got.double(), want, **tol), (M, N, K)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H, G, hd, vd", [(3, 2, 12, 20), (4, 1, 64, 32), (2, 2, 7, 7)])
def test_norms_over_the_projections_and_values_into_the_cache(dtype, H, G, hd, vd):
    from ferrox_amd import ops
    gen = torch.Generator().manual_seed(9)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    T, bs = 21, 8
    qkv = torch.randn(T, (H + G) * hd + G * vd + 3, generator=gen)
    wq, wk = (1 + 0.2 * torch.randn(H * hd, generator=gen)).to(dtype), (1 + 0.2 * torch.randn(G * hd, generator=gen)).to(dtype)
    pos = torch.arange(40, 40 + T, dtype=torch.int32)
    table = torch.randperm(10, generator=gen).to(torch.int32).view(1, -1)
    kp = torch.zeros(11, G, bs, hd, dtype=dtype, device="cuda")
    vp = torch.zeros(11, G, vd, bs, dtype=dtype, device="cuda")
    q_out = torch.zeros(T, H * hd, dtype=dtype, device="cuda")
    ops.span_norm_kv_write(qkv.cuda(), q_out, wq.cuda(), wk.cuda(), 1e-5, pos.cuda(), torch.zeros(T, dtype=torch.int32, device="cuda"),
                           table.cuda(), kp, vp, H, G, hd, bs, v_dim=vd)
    x = qkv.to(F64)
    assert float((q_out.cpu().to(F64) - plain.rms_norm(x[:, :H * hd], wq.to(F64), 1e-5)).abs().max()) < tol
    k_want = plain.rms_norm(x[:, H * hd:(H + G) * hd], wk.to(F64), 1e-5).view(T, G, hd)
    v_want = x[:, (H + G) * hd:(H + G) * hd + G * vd].view(T, G, vd)
    for t in range(T):
        page, slot = int(table[0, int(pos[t]) // bs]), int(pos[t]) % bs
        assert float((kp[page, :, slot].cpu().to(F64) - k_want[t]).abs().max()) < tol
        assert float((vp[page, :, :, slot].cpu().to(F64) - v_want[t]).abs().max()) < tol


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T, H, R, P, rot", [(37, 3, 24, 12, 8), (1, 16, 192, 64, 64), (5, 10, 33, 7, 6), (300, 2, 64, 16, 16), (4, 9, 20, 4, 0)])
def test_latents_and_query_heads_in_one_launch(dtype, T, H, R, P, rot):
    """The cache write that also turns the queries' heads: the pages are those of the launch without queries, the heads the
    plain formula's, their unrotated parts rounded once."""
    from ferrox_amd import ops
    gen = torch.Generator().manual_seed(T)
    freqs, mag = plain.rotation({"dims": rot, "base": 50.0, "scaling": dict(zip(("factor", "original", "fast", "slow"), u.STRETCH))}) if rot else ([], 1.0)
    n, bs = H * (R + P), 16
    down = torch.randn(T, n + R + P + 2, generator=gen).cuda()
    w = (1.0 + 0.2 * torch.randn(R, generator=gen)).to(dtype).cuda()
    pos = torch.tensor([400 + 3 * t for t in range(T)], dtype=torch.int32).cuda()
    n_pages = (400 + 3 * T) // bs + 2
    table = torch.randperm(n_pages, generator=gen).to(torch.int32).view(1, -1).cuda()
    seqs = torch.zeros(T, dtype=torch.int32, device="cuda")
    inv = ops.rotary_frequencies("cuda", rot, 50.0, tuple(freqs)) if rot else None
    pages = []
    for heads in (None, (down, H)):
        kp = torch.zeros(n_pages + 1, 1, bs, R + P, dtype=dtype, device="cuda")
        vp = torch.zeros(n_pages + 1, 1, R, bs, dtype=dtype, device="cuda")
        q = ops.latent_kv_write(down[:, n:], w, 1e-5, pos, seqs, table, kp, vp, R, P, rot, bs, inv, mag, q_heads=heads)
        pages.append((kp, vp))
    assert torch.equal(pages[0][0], pages[1][0]) and torch.equal(pages[0][1], pages[1][1])
    src = down[:, :n].cpu().view(T, H, R + P)
    got = q.view(T, H, R + P)
    assert torch.equal(got[..., :R].cpu(), src[..., :R].to(dtype)) and torch.equal(got[..., R + rot:].cpu(), src[..., R + rot:].to(dtype))
    want = src[..., R:R + rot].to(F64).clone()
    for t in range(T):
        for i, f in enumerate(freqs):
            a = float(torch.tensor(float(pos[t]), dtype=torch.float32) * torch.tensor(f, dtype=torch.float32))
            x, y = src[t, :, R + 2 * i].to(F64), src[t, :, R + 2 * i + 1].to(F64)
            want[t, :, 2 * i], want[t, :, 2 * i + 1] = (x * math.cos(a) - y * math.sin(a)) * mag, (y * math.cos(a) + x * math.sin(a)) * mag
    assert torch.allclose(got[..., R:R + rot].cpu().to(F64), want, **(dict(rtol=1e-5, atol=1e-5) if dtype == torch.float32 else dict(rtol=1e-2, atol=2e-2)))


def attention_reference(q, k, v, scale, window, bias, sinks, gate, softcap=0.0, slopes=None):
    """float64 attention of one sequence from position 0: q [n, H, D], k [n, G, D], v [n, G, V], bias [H, distances]."""
    n, H, _ = q.shape
    G = k.shape[1]
    see = plain.visible(n, window)
    dist = (torch.arange(n)[:, None] - torch.arange(n)[None, :]).clamp(min=0)
    out = torch.zeros(n, H, v.shape[2], dtype=F64)
    for h in range(H):
        s = (q[:, h].to(F64) @ k[:, h // (H // G)].to(F64).T) * scale
        if softcap:
            s = softcap * torch.tanh(s / softcap)
        if slopes is not None:
            s = s - float(slopes[h]) * dist
        s = (s + bias[h].to(F64)[dist.clamp(max=bias.shape[1] - 1)]).masked_fill(~see, -math.inf)
        top = s.max(-1, keepdim=True).values
        e = torch.exp(s - top)
        total = e.sum(-1, keepdim=True) + (torch.exp(sinks[h].to(F64) - top) if sinks is not None else 0.0)
        out[:, h] = (e / total) @ v[:, h // (H // G)].to(F64)
    if gate is not None:
        g = torch.sigmoid(gate.to(F64))
        out = out * (g.unsqueeze(-1) if g.shape[1] == H else g.view(n, H, -1))
    return out


@pytest.mark.parametrize("dtype,hd,vd,bs,G", [
    ("float32", 24, 24, 16, 2), ("bfloat16", 64, 64, 64, 2), ("bfloat16", 128, 128, 64, 1), ("bfloat16", 48, 48, 16, 2),
    ("bfloat16", 32, 32, 16, 4), ("bfloat16", 20, 20, 16, 2), ("bfloat16", 64, 128, 64, 2), ("bfloat16", 80, 64, 16, 1),
    ("bfloat16", 256, 192, 64, 1), ("bfloat16", 160, 160, 16, 2), ("bfloat16", 288, 256, 16, 1), ("float32", 320, 272, 64, 1)])
def test_attention_kernels_with_distance_biases(dtype, hd, vd, bs, G):
    """The attention kernels alone with a number per head and distance: tables that end before, at and behind the window,
    of one number, and too long for the copy in LDS; a constant sink, a float32 gate per head and per element, a cap and
    slopes beside the biases.  A prompt of 333 positions in scattered pages, read as one portion, as a portion deep in the
    sequence (by both item sizes where there are two) and as single queries."""
    from ferrox_amd import ops
    dt = getattr(torch, dtype)
    gen = torch.Generator().manual_seed(hd + vd)
    n, H = 333, 4
    q = torch.randn(n, H, hd, generator=gen).to(dt)
    k, v = torch.randn(n, G, hd, generator=gen).to(dt), torch.randn(n, G, vd, generator=gen).to(dt)
    gates = {"head": torch.randn(n, H, generator=gen), "element": torch.randn(n, H * vd, generator=gen)}
    zeros, learned = torch.zeros(H), torch.randn(H, generator=gen) + 1.0
    slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)])
    n_blocks = -(-n // bs)
    order = torch.randperm(n_blocks + 3, generator=gen)[:n_blocks].to(torch.int32)
    k_pages = torch.full((n_blocks + 3, G, bs, hd), float("nan")).to(dt)
    v_pages = torch.full((n_blocks + 3, G, vd, bs), float("nan")).to(dt)
    for t in range(n):
        k_pages[order[t // bs], :, t % bs] = k[t]
        v_pages[order[t // bs], :, :, t % bs] = v[t]
    qd, kp, vp = q.view(n, -1).cuda(), k_pages.cuda(), v_pages.cuda()
    positions = torch.arange(n, dtype=torch.int32, device="cuda")
    tol = 3e-5 if dtype == "float32" else 2.5e-2
    table = order.view(1, -1).cuda()
    item = lambda x: torch.tensor(x, dtype=torch.int32, device="cuda")      # noqa: E731
    for window, n_bias, sinks, gate, cap, slope in ((40, 40, zeros, None, 0.0, False), (100, 30, zeros, "head", 0.0, False),
                                                    (0, 150, None, "element", 0.0, False), (70, 1, learned, None, 1.5, True),
                                                    (0, 6200, zeros, "head", 0.0, False), (64, 64, None, None, 2.0, False)):
        bias = torch.randn(H, n_bias, generator=gen) * 2
        want = attention_reference(q, k, v, 0.2, window, bias, sinks, gates[gate] if gate else None, cap, slopes if slope else None).view(n, -1)
        common = (H, G, hd, bs, window, 0.2)
        extra = dict(v_dim=vd, sinks=sinks.cuda() if sinks is not None else None, gate=gates[gate].cuda() if gate else None,
                     gate_per_head=gate == "head", softcap=cap, slopes=slopes.cuda() if slope else None,
                     distance_bias=ops.distance_bias_rows(bias).cuda())
        for tile in sorted({64, ops.attention_tile_queries(dt, hd, bs) if vd == hd and n_bias < ops.BIAS_ROW_MAX else 64}):
            for first in (0, 200):
                starts = list(range(first, n, tile))
                out = torch.full((n, H * vd), float("nan"), dtype=dt, device="cuda")
                ops.attention_tiles(qd, out, kp, vp, table, positions, item([0] * len(starts)), item(starts),
                                    item([min(tile, n - s) for s in starts]), *common, tile_q=tile, **extra)
                err = (out[first:].cpu().to(F64) - want[first:]).abs().max()
                assert float(err) < tol, (window, n_bias, gate, tile, first, float(err))
        toks = [0, 1, 39, 40, 63, 64, 200, 263, 264, 332]
        for chunk in (None, 64):
            out = torch.full((n, H * vd), float("nan"), dtype=dt, device="cuda")
            ops.attention_decode(qd, out, kp, vp, table, positions, torch.zeros(len(toks), dtype=torch.int32, device="cuda"),
                                 item(toks), *common, max_kv_len=n, chunk=chunk, **extra)
            err = (out[toks].cpu().to(F64) - want[toks]).abs().max()
            assert float(err) < tol, (window, n_bias, gate, "decode", chunk, float(err))


# ---------------------------------------------------------------------------
# whole models: prompts, decoding, portions, batches
# ---------------------------------------------------------------------------
def main_requests():
    V = u.CFG_MAIN["vocab"]
    return {"r97": u.random_tokens(V, 97, 1), "r23": u.random_tokens(V, 23, 2), "r1": u.random_tokens(V, 1, 3),
            "r50": u.random_tokens(V, 50, 4), "r2": u.random_tokens(V, 2, 5)}


@pytest.mark.parametrize("dtype", DTYPES)
def test_whole_prompts_and_decoding(tmp_path_factory, dtype):
    weights, model = model_for(tmp_path_factory, "main", u.CFG_MAIN, 3, dtype)
    reqs = main_requests()
    run_and_check(u.CFG_MAIN, weights, model, reqs, [[(r, len(t))] for r, t in reqs.items()], dtype, "whole")
    # most of a prompt in one step, the last 40 tokens (or all but one) one by one: the windows of 5, 13 and 30 positions
    # pass over decoded tokens, across the page borders at 16, 32, ...
    sched = []
    for r, t in reqs.items():
        first = max(1, len(t) - 40)
        sched += [[(r, first)]] + [[(r, 1)]] * (len(t) - first)
    run_and_check(u.CFG_MAIN, weights, model, reqs, sched, dtype, "decode")
    one = {"r50": reqs["r50"]}
    run_and_check(u.CFG_MAIN, weights, model, one, [[("r50", 1)]] * 50, dtype, "token by token")


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_of_changing_size(tmp_path_factory, dtype):
    weights, model = model_for(tmp_path_factory, "main", u.CFG_MAIN, 3, dtype)
    reqs = main_requests()
    sizes = [2, 5, 2, 16, 1, 7, 24, 3, 2, 17, 1, 1, 9]
    sched = []
    for r, t in reqs.items():
        left, i = len(t), 0
        while left:
            n = min(sizes[i % len(sizes)], left)
            sched.append([(r, n)])
            left -= n
            i += 1
    run_and_check(u.CFG_MAIN, weights, model, reqs, sched, dtype, "portions")
    pairs = [[("r50", 2)]] * 25
    run_and_check(u.CFG_MAIN, weights, model, {"r50": reqs["r50"]}, pairs, dtype, "two at a time")


@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_batches_with_pages_and_slots_used_again(tmp_path_factory, dtype):
    """Up to three live requests under three slots and a pool of 14 pages of 16 (the requests' sum needs 18):
    portions beside single tokens, requests that pause, slots and pages taken again."""
    weights, model = model_for(tmp_path_factory, "main", u.CFG_MAIN, 3, dtype)
    reqs = main_requests()
    reqs["s40"] = u.random_tokens(u.CFG_MAIN["vocab"], 40, 7)
    sched = [
        [("r97", 30), ("r23", 2), ("r1", 1)],
        [("r97", 3), ("r23", 1), ("r2", 2)],                    # r1's slot goes to r2
        [("r97", 1), ("r23", 18)],
        [("r23", 1), ("r50", 21)],                              # r97 pauses
        [("r97", 40), ("r23", 1), ("r50", 1)],                  # r23 ends
        [("r97", 1), ("r50", 27), ("s40", 2)],
        [("r97", 22), ("r50", 1), ("s40", 37)],                 # r97 and r50 end
        [("s40", 1)],
    ]
    run_and_check(u.CFG_MAIN, weights, model, reqs, sched, dtype, "mixed", num_pages=14, max_seqs=3)
    got_alone, _ = u.run_schedule(runner_of(model, num_pages=14, max_seqs=3), reqs, [[(r, len(t))] for r, t in reqs.items()])
    got_mixed, _ = u.run_schedule(runner_of(model, num_pages=14, max_seqs=3), reqs, sched)
    for r in reqs:
        assert float(u.row_errors(got_mixed[r], got_alone[r]).max()) <= u.EDGE_LIMIT[dtype], r


def test_one_slot_for_requests_in_a_row(tmp_path_factory):
    """One slot and ten pages for 215 tokens: every request takes the slot and the pages that the one before left; pages of
    windows that have passed come back meanwhile."""
    weights, model = model_for(tmp_path_factory, "main", u.CFG_MAIN, 3, "float32")
    V = u.CFG_MAIN["vocab"]
    reqs = {"z": u.random_tokens(V, 150, 2), "y": u.random_tokens(V, 60, 3), "x": u.random_tokens(V, 5, 4)}
    sched = [[("z", 8)]] * 17 + [[("z", 1)]] * 14 + [[("y", 7)]] * 8 + [[("y", 2)]] * 2 + [[("x", 2)], [("x", 1)], [("x", 2)]]
    run_and_check(u.CFG_MAIN, weights, model, reqs, sched, "float32", "one slot", num_pages=10, max_seqs=1)


# ---------------------------------------------------------------------------
# where a fault hides behind random weights
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
def test_keys_at_window_edges_and_page_borders(tmp_path_factory, dtype):
    """The biases of the farthest distances are high and those near low, so the last key inside the window carries most of
    the output: a window one position off, a key lost at a page's border or a wrong row of the table moves the logits at
    every position.  A window of 40 over pages of 16; in the prompt, in portions cut at and beside the edges, and under
    decoded tokens."""
    cfg = u.config([u.attention_layer(heads=4, kv_heads=2, dim=16, vdim=16, scale=0.2, bias_max=38, window=40, mlp=u.dense(32))])

    def far_keys_first(w):
        t = torch.full((u.BIAS_ROWS, 4), -4.0)
        t[-1] = 3.0                                 # distances 38 and 39
        t[6] = torch.tensor([-4.0, 2.0, -4.0, 2.0])  # a few in the middle
        w["l0.mix.rel"] = t.to(torch.bfloat16)

    weights, model = model_for(tmp_path_factory, "edges", cfg, 21, dtype, change=far_keys_first)
    reqs = {"long": u.random_tokens(cfg["vocab"], 330, 6)}
    limit = u.EDGE_LIMIT[dtype]
    kw = dict(limit=limit, num_pages=30)
    run_and_check(cfg, weights, model, reqs, [[("long", 330)]], dtype, "edges whole", **kw)
    run_and_check(cfg, weights, model, reqs, [[("long", 235)]] + [[("long", 1)]] * 95, dtype, "edges decode", **kw)
    cut = [39, 2, 38, 1, 1, 40, 41, 38, 80, 2, 39, 9]
    run_and_check(cfg, weights, model, reqs, [[("long", n)] for n in cut], dtype, "edges portions", **kw)
    w = u.as_float64(weights)
    base = plain.forward(cfg, w, reqs["long"])
    for change in ({"mask": {"size": 39}}, {"mask": {"size": 41}}, {"bias_max": 36}):
        off = u.row_errors(plain.forward(u.changed(cfg, 0, **change), w, reqs["long"]), base)
        assert float(off.max()) > 3 * limit and int((off > limit).sum()) > 60, f"{change} would not show"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["latent", "latent_2"])
def test_a_far_key_among_hundreds(tmp_path_factory, dtype, kind):
    """The key of one early token stands out for the queries of another token (in the first head's unrotated part: the
    queries' rows there are made to meet W_uk c), 387 positions later too; with the early token changed the logits move."""
    second = kind == "latent_2"
    layer = (u.latent_layer_2 if second else u.latent_layer)(heads=2, dim=24, rot_dim=8, vdim=24, kv_rank=32, scale=0.2)
    cfg = u.config([layer], emb_scale=1.0)
    key_token, query_token = 17, 93

    def meet(w):
        g = torch.Generator().manual_seed(4)
        wf = {name: t.float() for name, t in w.items()}
        k_in, q_in = wf["embed"][key_token], wf["embed"][query_token]
        c = plain.rms_norm((wf["l0.mix.dkv"] @ k_in)[None, :32], wf["l0.mix.dkv.norm"], 1e-6)[0]
        direction = torch.randn(24, generator=g)
        direction = 8.0 * direction / direction.norm()
        uk = wf["l0.mix.uk"]
        uk[:24] += torch.outer(direction - uk[:24] @ c, c) / (c @ c)
        w["l0.mix.uk"] = uk.to(torch.bfloat16)
        if second:
            q_in = plain.rms_norm((wf["l0.mix.dq"] @ q_in)[None], wf["l0.mix.dq.norm"], 1e-6)[0]
        w["l0.norm1"] = (2.0 * wf["l0.norm1"]).to(torch.bfloat16)
        name = "l0.mix.uq" if second else "l0.mix.q"
        q = wf[name]
        q[:24] += torch.outer(direction - q[:24] @ q_in, q_in) / (q_in @ q_in)
        w[name] = q.to(torch.bfloat16)

    weights, model = model_for(tmp_path_factory, "far_" + kind, cfg, 2, dtype, change=meet)
    tokens = [t if t not in (key_token, query_token) else 5 for t in u.random_tokens(cfg["vocab"], 390, 8)]
    tokens[3] = key_token
    for p in (150, 255, 256, 340, 389):
        tokens[p] = query_token
    kw = dict(limit=u.EDGE_LIMIT[dtype], num_pages=40)
    run_and_check(cfg, weights, model, {"a": tokens}, [[("a", 390)]], dtype, "far whole", **kw)
    run_and_check(cfg, weights, model, {"a": tokens}, [[("a", 2)], [("a", 253)]] + [[("a", 1)]] * 20 + [[("a", 65)], [("a", 48)]] + [[("a", 1)]] * 2,
                  dtype, "far cut", **kw)
    w = u.as_float64(weights)
    base = plain.forward(cfg, w, tokens)
    other = list(tokens)
    other[3] = 5
    moved = u.row_errors(plain.forward(cfg, w, other), base)
    assert float(moved[[150, 255, 256, 340, 389]].min()) > 3 * u.EDGE_LIMIT[dtype], "the far key does not show"


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_sink_that_takes_nearly_all(tmp_path_factory, dtype):
    """Biases far below zero at most distances: the one in the denominator outweighs every key there, so outputs are small
    and their size carries what the norm behind them makes of it; without it they would be full averages."""
    cfg = u.config([u.attention_layer(heads=2, kv_heads=1, dim=16, vdim=16, bias_max=20, window=25), u.latent_layer_2()])

    def low(w):
        t = torch.full((u.BIAS_ROWS, 2), -6.0)
        t[:, 1] = -1.0
        w["l0.mix.rel"] = t.to(torch.bfloat16)

    weights, model = model_for(tmp_path_factory, "sink", cfg, 5, dtype, change=low)
    reqs = {"a": u.random_tokens(cfg["vocab"], 60, 1)}
    run_and_check(cfg, weights, model, reqs, [[("a", 40)]] + [[("a", 1)]] * 20, dtype, "sink", limit=u.EDGE_LIMIT[dtype])
    w = u.as_float64(weights)
    base = plain.forward(cfg, w, reqs["a"])
    w["l0.mix.rel"] = w["l0.mix.rel"] + 6.0            # (a constant on all scores: nothing without a sink)
    assert float(u.row_errors(plain.forward(cfg, w, reqs["a"]), base).max()) > 2 * u.EDGE_LIMIT["bfloat16"]


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_on_the_matrix_units(tmp_path_factory, dtype):
    """Sizes that take the bfloat16 kernels' matrix-unit paths (head sizes in multiples of 16, widths in multiples of
    64, pages of 64): a prompt, then 140 tokens one by one from recorded steps, two requests decoding side by side."""
    weights, model = model_for(tmp_path_factory, "mfma", u.CFG_MFMA, 17, dtype, bias_rows=16)
    reqs = {"x": u.random_tokens(u.CFG_MFMA["vocab"], 300, 3), "y": u.random_tokens(u.CFG_MFMA["vocab"], 150, 4)}
    kw = dict(block_size=64, num_pages=10)
    sched = [[("x", 160)], [("y", 10)]] + [[("x", 1), ("y", 1)]] * 140
    run_and_check(u.CFG_MFMA, weights, model, reqs, sched, dtype, "long decode", **kw)
    run_and_check(u.CFG_MFMA, weights, model, reqs, [[("x", 300), ("y", 150)]], dtype, "whole", **kw)
    cut = [[("x", 130), ("y", 3)], [("x", 2), ("y", 140)], [("x", 150), ("y", 7)], [("x", 18)]]
    run_and_check(u.CFG_MFMA, weights, model, reqs, cut, dtype, "portions", **kw)


def test_many_requests_decode_together(tmp_path_factory):
    """20 requests of unequal depth, filled up to a recorded size with stand-in rows."""
    weights, model = model_for(tmp_path_factory, "mfma", u.CFG_MFMA, 17, "bfloat16", bias_rows=16)
    V = u.CFG_MFMA["vocab"]
    reqs = {f"r{i}": u.random_tokens(V, 8 + i, 50 + i) for i in range(20)}
    sched = [[(r, len(t) - 6) for r, t in reqs.items()]] + [[(r, 1) for r in reqs]] * 6
    run_and_check(u.CFG_MFMA, weights, model, reqs, sched, "bfloat16", "twenty", block_size=64, num_pages=24, max_seqs=20)


@pytest.mark.parametrize("dtype", DTYPES)
def test_sizes_that_fit_no_vector(tmp_path_factory, dtype):
    """Head sizes, ranks, widths and a vocabulary that are no multiples of 16, 8 or 4: the kernels' guarded paths."""
    cfg = u.config([u.attention_layer(heads=3, kv_heads=3, dim=10, vdim=14, scale=0.4, bias_max=11, window=9, mlp=u.dense(30)),
                    u.latent_layer(heads=5, dim=6, rot_dim=10, vdim=7, kv_rank=21, rot_dims=6, mlp=u.dense(22)),
                    u.latent_layer_2(heads=7, dim=9, rot_dim=6, vdim=5, kv_rank=13, q_rank=11)], width=70, vocab=151)
    weights, model = model_for(tmp_path_factory, "odd", cfg, 13, dtype, bias_rows=6)
    reqs = {"a": u.random_tokens(151, 45, 1), "b": u.random_tokens(151, 20, 2)}
    sched = [[("a", 30), ("b", 2)], [("a", 1), ("b", 17)]] + [[("a", 1), ("b", 1)]] + [[("a", 1)]] * 13
    run_and_check(cfg, weights, model, reqs, sched, dtype, "odd sizes")


@pytest.mark.parametrize("dtype", DTYPES)
def test_latents_wider_than_the_matrix_units_heads(tmp_path_factory, dtype):
    cfg = u.config([u.latent_layer(heads=2, dim=16, rot_dim=32, vdim=16, kv_rank=272, base=1000.0),
                    u.latent_layer_2(heads=3, dim=16, rot_dim=16, vdim=24, kv_rank=160, q_rank=48)])
    weights, model = model_for(tmp_path_factory, "wide", cfg, 19, dtype)
    reqs = {"a": u.random_tokens(cfg["vocab"], 90, 1), "b": u.random_tokens(cfg["vocab"], 30, 2)}
    run_and_check(cfg, weights, model, reqs, [[("a", 70), ("b", 3)], [("b", 20), ("a", 1)]] + [[("a", 1), ("b", 1)]] * 7 + [[("a", 12)]],
                  dtype, "wide latents")


def test_a_recorded_step_replayed_equals_the_eager_one(tmp_path_factory):
    """Decode steps from a recording against the same steps launched kernel by kernel, with other work in between."""
    weights, model = model_for(tmp_path_factory, "main", u.CFG_MAIN, 3, "float32")
    tokens = u.random_tokens(u.CFG_MAIN["vocab"], 40, 12)
    outs = []
    for graphs in (True, False):
        runner = runner_of(model, use_graphs=graphs)
        got, _ = u.run_schedule(runner, {"a": tokens, "b": tokens[5:]}, [[("a", 20), ("b", 15)]] + [[("a", 1), ("b", 1)]] * 9
                                + [[("a", 2)], [("b", 3)]] + [[("a", 1), ("b", 1)]] * 8 + [[("a", 1)]])
        outs.append(got)
    for r in ("a", "b"):
        assert torch.equal(outs[0][r], outs[1][r])


# ---------------------------------------------------------------------------
# through the engine's own entry points: scheduler, sampling, recorded steps, command line, replay
# ---------------------------------------------------------------------------
def plain_greedy(cfg, weights, prompt, n):
    tokens, w = list(prompt), u.as_float64(weights)
    for _ in range(n):
        tokens.append(int(plain.forward(cfg, w, tokens)[-1].argmax()))
    return tokens[len(prompt):]


def test_greedy_generation_through_the_engine(tmp_path_factory):
    from ferrox_amd.engine.api import Engine
    weights, model = model_for(tmp_path_factory, "main", u.CFG_MAIN, 3, "float32")
    prompts = [u.random_tokens(u.CFG_MAIN["vocab"], n, 90 + n) for n in (3, 30, 1, 47)]
    want = [plain_greedy(u.CFG_MAIN, weights, p, 12) for p in prompts]
    assert len({t for w in want for t in w}) >= 6, "the expected continuations say too little"
    # steps of at most 16 tokens: prompts are cut into portions that run beside other requests' decoded tokens
    engine = Engine(model=model, block_size=16, num_pages=32, max_seqs=3, max_tokens_per_step=16, prefill_chunk=16)
    assert engine.generate(prompts, max_new_tokens=12, temperature=0.0, ignore_eos=True) == want
    # too few pages for all at once: requests wait, or are preempted and recomputed
    small = Engine(model=model, block_size=16, num_pages=6, max_seqs=4, max_tokens_per_step=32, prefill_chunk=32)
    assert small.generate(prompts, max_new_tokens=12, temperature=0.0, ignore_eos=True) == want


def test_command_line_and_replay(tmp_path_factory):
    import json
    import os
    import subprocess
    import sys

    import numpy as np
    from conftest import ROOT
    weights = u.make_weights(u.CFG_MAIN, 3)
    folder = u.write_model(str(tmp_path_factory.mktemp("zazerax_cli")), u.CFG_MAIN, weights)
    prompt = u.random_tokens(u.CFG_MAIN["vocab"], 9, 77)
    want = plain_greedy(u.CFG_MAIN, weights, prompt, 6)
    out = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "ferrox-amd"), "-m", folder, "--tokens",
                          ",".join(map(str, prompt)), "-n", "6", "--temp", "0", "--repeat-penalty", "1.0", "--ignore-eos", "--dtype", "float32",
                          "--block-size", "16", "--num-pages", "16"],
                         capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    assert ",".join(map(str, want)) in out.stdout.replace(" ", ""), (out.stdout[-500:], want)
    # random weights of the named shape, cut to three layers, through the command line
    out = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "ferrox-amd"), "--random-weights", "--config", "zazerax-2k", "--layers", "3",
                          "--tokens", "1,2,3,4,5", "-n", "4", "--temp", "0", "--ignore-eos", "--num-pages", "8"],
                         capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    # the step-by-step replay: two requests, a portion beside a single token, logits at chosen places
    a, b = u.random_tokens(u.CFG_MAIN["vocab"], 30, 1), u.random_tokens(u.CFG_MAIN["vocab"], 4, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:17], "want": [0, 16]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[17:29], "want": []}, {"id": "b", "tokens": b[:3], "want": [2]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[3:], "want": [0]}, {"id": "a", "tokens": a[29:], "want": [0]}], "end": ["a", "b"]}]
    out_dir = str(tmp_path_factory.mktemp("zazerax_replay"))
    run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
                          "--out", out_dir, "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                         capture_output=True, text=True, timeout=300)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [line for line in run.stdout.splitlines() if line.startswith("done")] == ["done 0", "done 1", "done 2"]
    w = u.as_float64(weights)
    la, lb = plain.forward(u.CFG_MAIN, w, a), plain.forward(u.CFG_MAIN, w, b)
    V = u.CFG_MAIN["vocab"]
    for step, want_rows in ((0, [la[0], la[16]]), (1, [lb[2]]), (2, [lb[3], la[29]])):
        got = torch.from_numpy(np.fromfile(os.path.join(out_dir, f"{step}.f32"), dtype="<f4").reshape(-1, V))
        assert float(u.row_errors(got, torch.stack(want_rows)).max()) <= u.LIMIT["float32"], step
