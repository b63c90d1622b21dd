"""Besulix on the GPU against the plain model (`plain_besulix`): every mechanism alone, the new kernels alone, whole
prompts, decoding through cache and state, portions down to two tokens, unequal batches, pages and slots used again,
keys just inside and outside chunk edges and at page borders in prompts and in decoding, the first tokens, states
written far back, long decoding, other sizes, and generation through the engine's entry points."""
import pytest
import torch

import besulix_util as u
import plain_besulix as plain

pytestmark = pytest.mark.gpu

_models = {}
F64 = torch.float64
DTYPES = ["float32", "bfloat16"]


def model_for(tmp_path_factory, name, cfg, seed, dtype, change=None, decay_rank=u.DECAY_RANK):
    """(weights as the plain model reads them, loaded engine model); made once per (name, dtype)."""
    from ferrox_amd.engine.loading import load_model
    key = (name, dtype)
    if key not in _models:
        weights = u.make_weights(cfg, seed, decay_rank)
        if change:
            change(weights)
        folder = u.write_model(str(tmp_path_factory.mktemp(f"besulix_{name}")), cfg, weights)
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
# each mechanism alone: models of one layer
# ---------------------------------------------------------------------------
SINGLE = {
    "memory": u.config([u.mlstm_layer()]),
    "memory_one_head": u.config([u.mlstm_layer(heads=1, dim=16, vdim=24, gate_cap=2.0)]),
    "memory_dense": u.config([u.mlstm_layer(mlp=u.dense(56, 0.4))]),
    "side_by_side": u.config([u.parallel_layer()]),
    "attention_alone": u.config([u.parallel_layer(heads=6, kv_heads=2, dim=16, vdim=16, right=0.0, left=1.0)]),
    "attention_one_key_head": u.config([u.parallel_layer(heads=5, kv_heads=1, dim=8, vdim=24, dims=2, chunk=11, right=0.0)]),
    "attention_wide_values_whole_rotation": u.config([u.parallel_layer(heads=2, kv_heads=2, dim=8, vdim=40, dims=8, base=20.0, chunk=16, right=0.0)]),
    "attention_nothing_rotated_in_keys": u.config([u.parallel_layer(dims=0, base=40.0, right=0.0)]),
    "attention_chunks_of_one": u.config([u.parallel_layer(chunk=1, right=0.0)]),
    "attention_one_chunk": u.config([u.parallel_layer(chunk=400, right=0.0)]),
    "time_mix_alone": u.config([u.parallel_layer(left=0.0, right=1.0)]),
    "time_mix_one_head": u.config([u.parallel_layer(r_heads=1, r_dim=40, left=0.0, right=-1.3)]),
    "time_mix_many_heads": u.config([u.parallel_layer(r_heads=12, r_dim=4, left=0.0)]),
    "one_token_of_vocabulary_cap": u.config([u.mlstm_layer(mlp=u.dense(24, 50.0))], softcap=0.5, eps=1e-3),
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

    def moved(**replace):
        return float(u.row_errors(plain.forward(cfg, dict(w, **replace), tokens), base).max())

    sight = u.EDGE_LIMIT["bfloat16"]
    assert moved(**{"l1.mix.left.sink": torch.full_like(w["l1.mix.left.sink"], -50.0)}) > sight
    assert moved(**{"l1.mix.left.temp": torch.ones_like(w["l1.mix.left.temp"])}) > 10 * u.EDGE_LIMIT["float32"]
    assert moved(**{"l2.mix.right.u": torch.zeros_like(w["l2.mix.right.u"])}) > sight
    assert moved(**{"l2.mix.right.w1": torch.zeros_like(w["l2.mix.right.w1"])}) > sight
    for s in "rkvgw":
        assert moved(**{f"l1.mix.right.mu.{s}": torch.zeros_like(w["l1.mix.right.mu.r"])}) > 10 * u.EDGE_LIMIT["float32"], s
    turn = plain.turn
    # values turned at the key but not back at the query, and not turned at all (the keys' rotation stays: it turns by
    # another function of the same name only where a head's first dimensions are taken)
    monkeypatch.setattr(plain, "turn", lambda x, pos, b, sign=1.0: x if sign < 0 else turn(x, pos, b, sign))
    assert moved() > sight
    monkeypatch.setattr(plain, "turn", lambda x, pos, b, sign=1.0: turn(x, pos, b, sign) if sign < 0 else x)
    assert moved() > sight


# ---------------------------------------------------------------------------
# the new kernels alone, against torch in float64
# ---------------------------------------------------------------------------
def starts_of(lengths):
    s = [0]
    for n in lengths:
        s.append(s[-1] + n)
    return torch.tensor(s, dtype=torch.int32, device="cuda")


def seqs_of(lengths):
    return torch.tensor([s for s, n in enumerate(lengths) for _ in range(n)], dtype=torch.int32, device="cuda")


@pytest.mark.parametrize("H, D, V, segments", [(3, 8, 12, 1), (2, 64, 64, 1), (1, 130, 33, 1), (2, 6, 5, 1), (2, 20, 24, 3), (1, 64, 40, 2),
                                               (2, 128, 16, 4), (1, 160, 8, 2)])
def test_outer_product_recurrence_with_a_decay_per_channel(H, D, V, segments):
    """Portions of unequal sequences in one launch, from states that an earlier launch left, whole and cut into
    segments (sequences shorter than a segment, ending inside the second, and filling all), against a loop."""
    from ferrox_amd import ops
    gen = torch.Generator().manual_seed(H * 100 + D)
    lengths, slots = ([37, 1, 9], [2, 0, 3]) if segments == 1 else ([65, 7, 64 * segments, 1], [2, 0, 3, 1])
    T = sum(lengths)
    q, k = (torch.randn(T, H * D, generator=gen) for _ in range(2))
    v = torch.randn(T, H * V, generator=gen)
    keep = torch.rand(T, H * D, generator=gen) * 0.6 + 0.4
    bonus = torch.randn(H, D, generator=gen)
    state0 = torch.randn(5, H, V, D, generator=gen)
    state = state0.clone().cuda()
    o = ops.channel_outer(q.cuda(), k.cuda(), v.cuda(), keep.cuda(), bonus.cuda(), state, starts_of(lengths),
                          torch.tensor(slots, dtype=torch.int32, device="cuda"), len(lengths), H, D, V, q_scale=0.7,
                          segments=segments).cpu().to(F64)
    t0 = 0
    for n, slot in zip(lengths, slots):
        S = state0[slot].to(F64).clone()                               # [H, V, D]
        for t in range(t0, t0 + n):
            qq, kk, dd = (x[t].to(F64).view(H, D) for x in (q, k, keep))
            kv = v[t].to(F64).view(H, V)[:, :, None] * kk[:, None, :]
            want = 0.7 * torch.einsum("hvd,hd->hv", S + bonus.to(F64)[:, None, :] * kv, qq)
            assert torch.allclose(o[t].view(H, V), want, rtol=2e-5, atol=5e-5), (t, n)
            S = dd[:, None, :] * S + kv
        assert torch.allclose(state[slot].cpu().to(F64), S, rtol=2e-5, atol=2e-5), n
        t0 += n
    assert torch.equal(state[4].cpu(), state0[4]), "a slot of no sequence was written"


@pytest.mark.parametrize("H, G, D, V, segments", [(2, 1, 20, 7, 3), (1, 1, 128, 64, 2), (2, 2, 64, 33, 5), (1, 1, 136, 9, 2)])
def test_outer_product_recurrence_in_segments(H, G, D, V, segments):
    """Factors per head with a normaliser: a cut portion against the same portion in one piece, and its pieces one after
    the other."""
    from ferrox_amd import ops
    gen = torch.Generator().manual_seed(D)
    lengths, slots = [64 * segments - 5, 3, 130], [1, 2, 0]
    T = sum(lengths)
    q, k = (torch.randn(T, G * D, generator=gen).cuda() for _ in range(2))
    v = torch.randn(T, H * V, generator=gen).cuda()
    keep, take = (torch.rand(T, H, generator=gen) * 0.4 + 0.6).cuda(), (torch.rand(T, H, generator=gen) + 0.2).cuda()
    state0 = torch.randn(3, H, V + 1, D, generator=gen).cuda()
    ids = torch.tensor(slots, dtype=torch.int32, device="cuda")
    a, b = state0.clone(), state0.clone()
    o1, n1 = ops.gated_outer(q, k, v, keep, take, a, starts_of(lengths), ids, 3, H, G, D, V, q_scale=0.3, normalizer=True, segments=1)
    o2, n2 = ops.gated_outer(q, k, v, keep, take, b, starts_of(lengths), ids, 3, H, G, D, V, q_scale=0.3, normalizer=True, segments=segments)
    for x, y in ((o1, o2), (n1, n2), (a, b)):
        assert torch.allclose(x, y, rtol=1e-4, atol=2e-5 * float(x.abs().max()))
    const = keep[0].contiguous()
    c, d = state0[:, :, :V].clone().contiguous(), state0[:, :, :V].clone().contiguous()
    o1 = ops.gated_outer(q, k, v, const, None, c, starts_of(lengths), ids, 3, H, G, D, V, segments=1)
    o2 = ops.gated_outer(q, k, v, const, None, d, starts_of(lengths), ids, 3, H, G, D, V, segments=segments)
    assert torch.allclose(o1, o2, rtol=1e-4, atol=2e-5 * float(o1.abs().max())) and torch.allclose(c, d, rtol=1e-4, atol=1e-4)


def test_segments_are_chosen_for_long_portions():
    from ferrox_amd import ops
    f, _ = ops._fn("recurrent", "fx_outer_segments")
    assert f(1, 32, 64, 64, 0, 200) == 1 and f(4, 32, 64, 64, 0, 1) == 1
    assert f(1, 32, 64, 64, 0, 2048) > 1 and f(1, 4, 64, 64, 0, 300) == 4      # (none shorter than 64 tokens)
    assert f(1, 4, 66, 64, 0, 3000) == 1, "key sizes that fit no vector run in one piece"
    assert f(64, 32, 128, 128, 1, 4096) == 4


def test_the_gates_scan_gives_the_same_bits_from_one_wave_and_many():
    from ferrox_amd import ops
    gen = torch.Generator().manual_seed(5)
    H, cap, lengths = 3, 4.0, [2100, 1, 64, 65, 1024]
    T = sum(lengths)
    xi, xf = (torch.randn(T, H, generator=gen) * 6).cuda(), (torch.randn(T, H, generator=gen) * 6 + 2).cuda()
    ids = torch.tensor([1, 3, 0, 2, 4], dtype=torch.int32, device="cuda")
    outs = []
    for longest in (1, max(lengths)):
        state = torch.randn(5, H, generator=torch.Generator().manual_seed(1)).cuda()
        outs.append((*ops.exp_gate_scan(xi, xf, cap, state, starts_of(lengths), ids, 5, H, longest=longest), state))
    for x, y in zip(*outs):
        assert torch.equal(x, y)
    mx = torch.randn(5, H, generator=torch.Generator().manual_seed(1)).to(F64)[1]
    for t in range(2100):                           # the first sequence, slot 1, against a loop
        i, f = cap * torch.tanh(xi[t].cpu().to(F64) / cap), plain.logsigmoid(cap * torch.tanh(xf[t].cpu().to(F64) / cap))
        new = torch.maximum(f + mx, i)
        assert torch.allclose(outs[1][2][t].cpu().to(F64), new, rtol=1e-5, atol=2e-5), t
        mx = new


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("C", [64, 37, 2056])
def test_token_shift(dtype, C):
    from ferrox_amd import ops
    gen = torch.Generator().manual_seed(C)
    lengths, slots = [6, 1, 11, 1], [1, 4, 0, 2]
    T = sum(lengths)
    x = torch.randn(T, C + 8, generator=gen).to(dtype)[:, :C]
    mu = torch.rand(3, C, generator=gen)
    state0 = torch.randn(5, C, generator=gen)
    state = state0.clone().cuda()
    wide = torch.zeros(T, C + 8, dtype=dtype, device="cuda")          # (rows further apart than they are long)
    wide[:, :C] = x.cuda()
    got = ops.token_shift(wide[:, :C], mu.cuda(), state, seqs_of(lengths), starts_of(lengths),
                          torch.tensor(slots, dtype=torch.int32, device="cuda")).cpu().to(F64)
    t0 = 0
    for n, slot in zip(lengths, slots):
        rows = x[t0:t0 + n].to(F64)
        before = torch.cat([state0[slot].to(F64)[None], rows[:-1]])
        for i in range(3):
            want = rows + (before - rows) * mu[i].to(F64)
            tol = dict(rtol=1e-5, atol=1e-5) if dtype == torch.float32 else dict(rtol=1e-2, atol=2e-2)
            assert torch.allclose(got[i, t0:t0 + n], want, **tol), (n, i)
        assert torch.equal(state[slot].cpu(), x[t0 + n - 1].float()), "the last row is carried"
        t0 += n
    assert torch.equal(state[3].cpu(), state0[3]), "a slot of no sequence was written"


@pytest.mark.parametrize("T, R, N", [(1, 5, 40), (7, 16, 256), (65, 64, 1028), (130, 3, 37), (100, 300, 72), (513, 130, 2048)])
def test_low_rank_decay(T, R, N):
    from ferrox_amd import ops
    gen = torch.Generator().manual_seed(T)
    low = torch.randn(T, R + 3, generator=gen)
    w2, w0 = torch.randn(N, R, generator=gen) / R ** 0.5, torch.randn(N, generator=gen) - 2
    got = ops.lowrank_decay(low.cuda()[:, :R], w2.t().contiguous().cuda(), w0.cuda())
    want = torch.exp(-torch.exp(torch.tanh(low[:, :R].to(F64)) @ w2.to(F64).T + w0.to(F64)))
    assert torch.allclose(got.cpu().to(F64), want, rtol=2e-5, atol=1e-6)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H", [70, 4500])
def test_normed_embedding(dtype, H):
    from ferrox_amd import ops
    gen = torch.Generator().manual_seed(H)
    table, w = torch.randn(20, H, generator=gen).to(dtype), torch.randn(H, generator=gen).to(dtype)
    ids = torch.tensor([3, 19, 0, 3], dtype=torch.int32)
    got = ops.embed_rmsnorm(table.cuda(), ids.cuda(), w.cuda(), 1e-3, scale=0.5)
    want = plain.rms_norm(0.5 * table.to(F64)[ids.long()], w.to(F64), 1e-3)
    assert torch.allclose(got.cpu().to(F64), want, rtol=1e-5, atol=1e-6)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_capped_products_of_every_kind_of_kernel(dtype):
    """The cap in the epilogues of the products for few rows, many rows, sizes that fit no vector, and very many columns."""
    from ferrox_amd import ops
    gen = torch.Generator().manual_seed(7)
    for M, N, K in ((3, 200, 64), (300, 384, 128), (33, 70, 52), (70, 1000, 256), (20, 66000, 64)):
        a, w = torch.randn(M, K, generator=gen).to(dtype).cuda(), (torch.randn(N, K, generator=gen) / K ** 0.5 * 4).to(dtype).cuda()
        got = ops.gemm(a, w, epilogue=ops.EPI_STORE_F32, store_activation="softcap", activation_params=(3.0, 0.0))
        z = a.float() @ w.float().t()
        assert torch.allclose(got, 3.0 * torch.tanh(z / 3.0), rtol=1e-4, atol=1e-4), (M, N, K)


def test_narrow_outputs_of_many_rows():
    """Few weight rows under many rows take the product for few rows: the tiled product's values."""
    from ferrox_amd import debug, ops
    gen = torch.Generator().manual_seed(9)
    for M, N, K in ((300, 16, 64), (2048, 64, 256), (1000, 130, 192), (257, 9, 72)):
        a, w = torch.randn(M, K, generator=gen).bfloat16().cuda(), torch.randn(N, K, generator=gen).bfloat16().cuda()
        want = a.double() @ w.double().t()
        got = ops.gemm(a, w, epilogue=ops.EPI_STORE_F32)
        assert torch.allclose(got.double(), want, rtol=1e-4, atol=1e-3), (M, N, K)
        with debug.kernel_switch("gemm", "plain_rows", 64):
            assert torch.allclose(ops.gemm(a, w, epilogue=ops.EPI_STORE_F32).double(), want, rtol=1e-4, atol=1e-3)


def turned(x, positions, base, sign=1.0):
    """Neighbouring pairs of x [T, heads, dims] turned by their positions (the layout the pages hold)."""
    n = x.shape[-1]
    halves = torch.cat([x[..., 0::2], x[..., 1::2]], dim=-1)
    y = plain.turn(halves, positions, base, sign)
    return torch.stack([y[..., :n // 2], y[..., n // 2:]], dim=-1).reshape(x.shape)


@pytest.mark.parametrize("dtype, nh, nkv, hd, vd, bs, rot, inter", [
    (torch.float32, 4, 2, 8, 12, 16, 4, False), (torch.bfloat16, 4, 1, 64, 64, 64, 64, False), (torch.bfloat16, 2, 2, 24, 40, 16, 10, True),
    (torch.float32, 3, 3, 130, 200, 8, 130, False), (torch.bfloat16, 3, 3, 32, 6, 16, 0, False)])
def test_turned_keys_and_values_into_the_cache(dtype, nh, nkv, hd, vd, bs, rot, inter):
    from ferrox_amd import ops
    gen = torch.Generator().manual_seed(nh + hd)
    positions = torch.tensor(list(range(29, 29 + 21)) + [0, 7])            # a portion across page borders, two single tokens
    seqs = [0] * 21 + [1, 2]
    T, base = len(seqs), 300.0
    qkv = torch.randn(T, (nh + nkv) * hd + nkv * vd, generator=gen)
    temp = torch.rand(nh, generator=gen) + 0.5
    table = torch.tensor([[3, 5, 1, 6, 7, 8, 9], [2] + [0] * 6, [4] + [0] * 6], dtype=torch.int32, device="cuda")
    k_pages = torch.zeros(10, nkv, bs, hd, dtype=dtype, device="cuda")
    v_pages = torch.zeros(10, nkv, vd, bs, dtype=dtype, device="cuda")
    q_out = torch.zeros(T, nh * hd, dtype=dtype, device="cuda")
    pos32 = positions.to(torch.int32).cuda()
    qk_turns = ops.angle_table(pos32, T, ops.rotary_frequencies("cuda", rot, base)) if rot else None
    v_turns = ops.angle_table(pos32, T, ops.rotary_frequencies("cuda", vd, base))
    ops.turned_kv_write(qkv.cuda(), q_out, pos32, torch.tensor(seqs, dtype=torch.int32, device="cuda"), table, k_pages, v_pages, nh, nkv,
                        hd, vd, bs, rot, inter, qk_turns, v_turns, temp.cuda())
    x = qkv.to(F64)
    rotate = (lambda y: torch.cat([turned(y[..., :rot], positions, base), y[..., rot:]], -1)) if inter \
        else (lambda y: plain.rotary(y, positions, base, rot)) if rot else (lambda y: y)
    q = rotate(x[:, :nh * hd].view(T, nh, hd)) * temp.to(F64)[:, None]
    k = rotate(x[:, nh * hd:(nh + nkv) * hd].view(T, nkv, hd))
    v = turned(x[:, (nh + nkv) * hd:].view(T, nkv, vd), positions, base)
    tol = dict(rtol=1e-5, atol=3e-5) if dtype == torch.float32 else dict(rtol=1e-2, atol=2e-2)
    assert torch.allclose(q_out.cpu().to(F64), q.reshape(T, nh * hd), **tol)
    for t, (p, s) in enumerate(zip(positions.tolist(), seqs)):
        page = int(table[s, p // bs])
        assert torch.allclose(k_pages[page, :, p % bs, :].cpu().to(F64), k[t], **tol), t
        assert torch.allclose(v_pages[page, :, :, p % bs].cpu().to(F64), v[t], **tol), t


@pytest.mark.parametrize("dtype, nh, nkv, hd, vd, bs", [
    (torch.float32, 4, 2, 16, 12, 16), (torch.bfloat16, 3, 1, 24, 10, 16), (torch.bfloat16, 4, 2, 32, 32, 16),
    (torch.bfloat16, 6, 2, 64, 64, 64), (torch.bfloat16, 4, 1, 128, 128, 64), (torch.bfloat16, 4, 2, 128, 80, 64),
    (torch.bfloat16, 5, 1, 192, 128, 64), (torch.bfloat16, 3, 3, 256, 256, 64)])
def test_outputs_turned_back_in_every_attention_kernel(dtype, nh, nkv, hd, vd, bs):
    """With and without the turn on the same queries and pages: portions by both item sizes, single queries by blocks of
    one and several waves, in one chunk of keys and in several with a merge; sinks and a chunked mask beside it."""
    from ferrox_amd import ops
    gen = torch.Generator().manual_seed(hd + vd)
    n_kv, base, chunk = 300, 50.0, 130
    pages = -(-n_kv // bs)
    k_pages = (torch.randn(pages + 1, nkv, bs, hd, generator=gen)).to(dtype).cuda()
    v_pages = (torch.randn(pages + 1, nkv, vd, bs, generator=gen)).to(dtype).cuda()
    table = torch.arange(1, pages + 1, dtype=torch.int32, device="cuda")[None].contiguous()
    sinks = torch.randn(nh, generator=gen).cuda()
    common = (nh, nkv, hd, bs, None, hd ** -0.5)
    tol = dict(rtol=1e-4, atol=1e-5) if dtype == torch.float32 else dict(rtol=2e-2, atol=2e-2)

    def compare(run, positions):
        T = len(positions)
        q = torch.randn(T, nh * hd, generator=gen).to(dtype).cuda()
        pos = torch.tensor(positions, dtype=torch.int32, device="cuda")
        turns = ops.angle_table(pos, T, ops.rotary_frequencies("cuda", vd, base))
        outs = []
        for tn in (None, turns):
            out = torch.full((T, nh * vd), float("nan"), dtype=dtype, device="cuda")
            run(q, out, pos, tn)
            outs.append(out.cpu().to(F64).view(T, nh, vd))
        want = turned(outs[0], torch.tensor(positions), base, sign=-1.0)
        assert torch.allclose(outs[1], want, **tol), float((outs[1] - want).abs().max())

    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device="cuda")
    extra = dict(mask_chunk=chunk, v_dim=vd, sinks=sinks)
    widest = ops.attention_tile_queries(dtype, hd, bs) if vd == hd else 64
    for tile in sorted({64, widest}):
        for first, n in ((0, n_kv), (100, 77), (n_kv - 2, 2)):
            items = [(t0, min(tile, n - t0)) for t0 in range(0, n, tile)]
            compare(lambda q, out, pos, tn: ops.attention_tiles(q, out, k_pages, v_pages, table, pos, i32([0] * len(items)),
                                                                i32([t for t, _ in items]), i32([m for _, m in items]), *common,
                                                                tile_q=tile, turns=tn, **extra), list(range(first, first + n)))
    singles = [0, 5, 129, 130, 131, 299]
    tables = table.expand(len(singles), -1).contiguous()
    for waves, split in ((0, None), (1, 512), (4, 512), (0, 64), (1, 64)):
        compare(lambda q, out, pos, tn: ops.attention_decode(q, out, k_pages, v_pages, tables, pos, i32(list(range(len(singles)))),
                                                             i32(list(range(len(singles)))), *common, max_kv_len=n_kv, chunk=split,
                                                             waves=waves, turns=tn, **extra), singles)


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
    # most of a prompt in one step, the last 40 tokens (or all but one) one by one: states and the last row are carried
    # on, chunks of 7, 24 and 50 end under decoded tokens, keys cross the page borders at 16, 32, ...
    sched = []
    for r, t in reqs.items():
        first = max(1, len(t) - 40)
        sched += [[(r, first)]] + [[(r, 1)]] * (len(t) - first)
    run_and_check(u.CFG_MAIN, weights, model, reqs, sched, dtype, "decode")
    # token by token from the first token on: states that start at zero, a token before the first that is zeros
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
    portions beside single tokens, requests that pause, slots (and the states in them) and pages taken again."""
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
    alone = runner_of(model, num_pages=14, max_seqs=3)
    mixed = runner_of(model, num_pages=14, max_seqs=3)
    got_alone, _ = u.run_schedule(alone, reqs, [[(r, len(t))] for r, t in reqs.items()])
    got_mixed, _ = u.run_schedule(mixed, reqs, sched)
    for r in reqs:
        assert float(u.row_errors(got_mixed[r], got_alone[r]).max()) <= u.EDGE_LIMIT[dtype], r


def test_one_slot_for_requests_in_a_row(tmp_path_factory):
    """One slot and six pages for 150 tokens: pages of chunks that have ended come back; every request takes the slot,
    the states, the carried row and the pages that the one before left."""
    weights, model = model_for(tmp_path_factory, "main", u.CFG_MAIN, 3, "float32")
    V = u.CFG_MAIN["vocab"]
    reqs = {"z": u.random_tokens(V, 150, 2), "y": u.random_tokens(V, 60, 3), "x": u.random_tokens(V, 5, 4)}
    sched = [[("z", 8)]] * 17 + [[("z", 1)]] * 14 + [[("y", 7)]] * 8 + [[("y", 2)]] * 2 + [[("x", 2)], [("x", 1)], [("x", 2)]]
    run_and_check(u.CFG_MAIN, weights, model, reqs, sched, "float32", "one slot", num_pages=6, max_seqs=1)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_prompt_in_segments_of_the_recurrences(tmp_path_factory, dtype):
    """700 tokens at once (the recurrences cut them into segments), then decoded tokens; beside it the same prompt in
    portions that are cut into other segments or none."""
    cfg = u.config([u.parallel_layer(chunk=130, r_heads=2, r_dim=16), u.mlstm_layer(heads=2, dim=16, vdim=20)], width=64)
    weights, model = model_for(tmp_path_factory, "segments", cfg, 5, dtype)
    from ferrox_amd import ops
    f, _ = ops._fn("recurrent", "fx_outer_segments")
    assert f(1, 2, 16, 16, 0, 700) > 2, "this prompt was meant to be cut"
    reqs = {"a": u.random_tokens(cfg["vocab"], 720, 4), "b": u.random_tokens(cfg["vocab"], 90, 5)}
    kw = dict(num_pages=60, limit=u.EDGE_LIMIT[dtype])
    run_and_check(cfg, weights, model, reqs, [[("a", 700), ("b", 70)]] + [[("a", 1), ("b", 1)]] * 20, dtype, "segments", **kw)
    run_and_check(cfg, weights, model, reqs, [[("a", 300)], [("b", 90), ("a", 101)], [("a", 319)]], dtype, "other segments", **kw)


# ---------------------------------------------------------------------------
# where a fault hides behind random weights
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
def test_keys_at_chunk_edges_and_page_borders(tmp_path_factory, dtype):
    """Queries and keys scaled up and sinks low: the softmax is peaked, so single keys carry the output, and a key that is
    lost or seen by mistake (a chunk's first or last position, a page's first or last slot, a key a chunk's length
    back, the query's own) moves the logits.  Chunks of 40 end inside pages of 16 and at their borders, in the prompt,
    in portions cut at and beside the edges, and under decoded tokens."""
    cfg = u.config([u.parallel_layer(heads=4, kv_heads=2, dim=16, vdim=16, scale=0.25, dims=8, chunk=40, r_heads=2, r_dim=8, left=1.0,
                                     right=0.3, mlp=u.dense(32))], width=64)
    # (bfloat16 rounds the scores themselves, a 250th of their size: scores of some tens would differ by tenths)
    factor = 5 if dtype == "float32" else 2.2

    def peaked(w):
        for name in ("q", "k", "q.b", "k.b"):
            w["l0.mix.left." + name] = (w["l0.mix.left." + name].float() * factor).to(torch.bfloat16)
        w["l0.mix.left.sink"] = torch.full_like(w["l0.mix.left.sink"], -2.0)

    weights, model = model_for(tmp_path_factory, "peaked", cfg, 21, dtype, change=peaked)
    reqs = {"long": u.random_tokens(cfg["vocab"], 330, 6)}
    limit = u.EDGE_LIMIT[dtype]
    kw = dict(limit=limit, num_pages=30)
    run_and_check(cfg, weights, model, reqs, [[("long", 330)]], dtype, "peaked whole", **kw)
    run_and_check(cfg, weights, model, reqs, [[("long", 235)]] + [[("long", 1)]] * 95, dtype, "peaked decode", **kw)
    cut = [39, 2, 38, 1, 1, 40, 41, 38, 80, 2, 39, 9]
    run_and_check(cfg, weights, model, reqs, [[("long", n)] for n in cut], dtype, "peaked portions", **kw)
    w = u.as_float64(weights)
    base = plain.forward(cfg, w, reqs["long"])
    for size in (39, 41):
        off = u.row_errors(plain.forward(u.changed(cfg, 0, left__mask={"size": size}), w, reqs["long"]), base)
        assert float(off.max()) > 3 * limit and int((off > limit).sum()) > 100, "chunks one position off would not show"


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_far_key_among_hundreds(tmp_path_factory, dtype):
    """One chunk of 400 positions: the key of one early token stands out for the queries of another token (their
    embeddings are made to meet in the first head's dimensions that are not rotated), and the value it hands over is
    turned by the distance."""
    cfg = u.config([u.parallel_layer(heads=2, kv_heads=2, dim=24, vdim=24, scale=0.2, dims=8, chunk=400, r_heads=1, r_dim=8, left=2.0,
                                     right=0.1)], width=64, vocab=150)
    W, key_token, query_token = 64, 17, 93

    def meet(w):
        g = torch.Generator().manual_seed(4)
        direction = torch.randn(24, generator=g)
        direction[:8] = 0                              # (the rotated dimensions stay out of it)
        direction = 8.0 * direction / direction.norm()
        for name, token in (("k", key_token), ("q", query_token)):
            e = w["embed"][token].float()
            h = e / e.pow(2).mean().sqrt() * w["embed.norm"].float()
            h = h / h.pow(2).mean().sqrt() * w["l0.norm1"].float()
            m = w["l0.mix.left." + name].float()
            m[:24] += torch.outer(direction - m[:24] @ h, h) / (h @ h)
            w["l0.mix.left." + name] = m.to(torch.bfloat16)

    weights, model = model_for(tmp_path_factory, "far_key", cfg, 2, dtype, change=meet)
    tokens = [t if t not in (key_token, query_token) else 5 for t in u.random_tokens(cfg["vocab"], 390, 8)]
    tokens[3] = key_token
    for p in (150, 255, 256, 340, 389):
        tokens[p] = query_token
    reqs = {"a": tokens}
    kw = dict(limit=u.EDGE_LIMIT[dtype], num_pages=40)
    run_and_check(cfg, weights, model, reqs, [[("a", 390)]], dtype, "far whole", **kw)
    run_and_check(cfg, weights, model, reqs, [[("a", 2)], [("a", 253)]] + [[("a", 1)]] * 20 + [[("a", 65)], [("a", 48)]] + [[("a", 1)]] * 2,
                  dtype, "far cut", **kw)
    w = u.as_float64(weights)
    base = plain.forward(cfg, w, tokens)
    other = list(tokens)
    other[3] = 5
    moved = u.row_errors(plain.forward(cfg, w, other), base)
    assert float(moved[[150, 256, 340, 389]].min()) > 3 * u.EDGE_LIMIT[dtype], "the far key does not show"


def test_a_state_written_far_back(tmp_path_factory):
    """Heads that hardly forget (a forget gate near one, decays near one): what token 3 wrote is read 200 tokens later,
    through portions and decoded tokens; with the token changed the last logits move."""
    cfg = u.config([u.mlstm_layer(heads=2, dim=8, vdim=8), u.parallel_layer(chunk=5, r_heads=2, r_dim=8, left=0.3, right=1.5)], width=32)

    def slow(w):
        w["l0.mix.f.b"] = torch.full_like(w["l0.mix.f.b"], 9.0)
        w["l1.mix.right.w0"] = torch.full_like(w["l1.mix.right.w0"], -9.0)

    weights, model = model_for(tmp_path_factory, "far_state", cfg, 9, "float32", change=slow)
    tokens = u.random_tokens(cfg["vocab"], 210, 8)
    sched = [[("a", 2)], [("a", 60)], [("a", 1)], [("a", 100)]] + [[("a", 1)]] * 47
    run_and_check(cfg, weights, model, {"a": tokens}, sched, "float32", "far state", limit=u.EDGE_LIMIT["float32"])
    w = u.as_float64(weights)
    other = list(tokens)
    other[3] = (other[3] + 1) % cfg["vocab"]
    moved = u.row_errors(plain.forward(cfg, w, other)[-1:], plain.forward(cfg, w, tokens)[-1:])
    assert float(moved) > 100 * u.LIMIT["float32"], "the last token does not see the third"


def test_channels_that_forget_at_once_and_never(tmp_path_factory):
    """Decays of exp(-exp(4)) (zero in float32) beside decays that round to one, in one head."""
    cfg = u.config([u.parallel_layer(left=0.2, right=1.0, r_heads=2, r_dim=8)])

    def extreme(w):
        t = torch.full((16,), -20.0)
        t[::2] = 4.0
        w["l0.mix.right.w0"] = t.to(torch.bfloat16)

    weights, model = model_for(tmp_path_factory, "extreme", cfg, 7, "float32", change=extreme)
    reqs = {"a": u.random_tokens(cfg["vocab"], 400, 1)}
    run_and_check(cfg, weights, model, reqs, [[("a", 390)]] + [[("a", 1)]] * 10, "float32", "extreme decays", limit=u.EDGE_LIMIT["float32"],
                  num_pages=30)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_on_the_matrix_units(tmp_path_factory, dtype):
    """Sizes that take the bfloat16 kernels' matrix-unit paths (head sizes in multiples of 16, widths in multiples of
    64, pages of 64): a prompt, then 140 tokens one by one from recorded steps, two requests decoding side by side."""
    weights, model = model_for(tmp_path_factory, "mfma", u.CFG_MFMA, 17, dtype, decay_rank=24)
    reqs = {"x": u.random_tokens(u.CFG_MFMA["vocab"], 300, 3), "y": u.random_tokens(u.CFG_MFMA["vocab"], 150, 4)}
    kw = dict(block_size=64, num_pages=10)
    sched = [[("x", 160)], [("y", 10)]] + [[("x", 1), ("y", 1)]] * 140
    run_and_check(u.CFG_MFMA, weights, model, reqs, sched, dtype, "long decode", **kw)
    run_and_check(u.CFG_MFMA, weights, model, reqs, [[("x", 300), ("y", 150)]], dtype, "whole", **kw)
    cut = [[("x", 130), ("y", 3)], [("x", 2), ("y", 140)], [("x", 150), ("y", 7)], [("x", 18)]]
    run_and_check(u.CFG_MFMA, weights, model, reqs, cut, dtype, "portions", **kw)


def test_many_requests_decode_together(tmp_path_factory):
    """Batches beyond the sizes whose projections go unsorted into the grouped product: 20 requests of unequal depth,
    filled up to a recorded size with stand-in rows."""
    weights, model = model_for(tmp_path_factory, "mfma", u.CFG_MFMA, 17, "bfloat16", decay_rank=24)
    V = u.CFG_MFMA["vocab"]
    reqs = {f"r{i}": u.random_tokens(V, 8 + i, 50 + i) for i in range(20)}
    sched = [[(r, len(t) - 6) for r, t in reqs.items()]] + [[(r, 1) for r in reqs]] * 6
    run_and_check(u.CFG_MFMA, weights, model, reqs, sched, "bfloat16", "twenty", block_size=64, num_pages=24, max_seqs=20)


@pytest.mark.parametrize("dtype", DTYPES)
def test_sizes_that_fit_no_vector(tmp_path_factory, dtype):
    """Head sizes, widths and a vocabulary that are no multiples of 16, 8 or 4: the kernels' guarded paths."""
    cfg = u.config([u.parallel_layer(heads=3, kv_heads=3, dim=10, vdim=14, scale=0.4, dims=6, chunk=9, r_heads=5, r_dim=6, mlp=u.dense(30, 0.9)),
                    u.mlstm_layer(heads=5, dim=6, vdim=10, mlp=u.dense(22, 2.0)),
                    u.parallel_layer(heads=7, kv_heads=1, dim=18, vdim=6, scale=0.3, dims=18, chunk=33, r_heads=1, r_dim=7)], width=70, vocab=151)
    weights, model = model_for(tmp_path_factory, "odd", cfg, 13, dtype, decay_rank=3)
    reqs = {"a": u.random_tokens(151, 45, 1), "b": u.random_tokens(151, 20, 2)}
    sched = [[("a", 30), ("b", 2)], [("a", 1), ("b", 17)]] + [[("a", 1), ("b", 1)]] + [[("a", 1)]] * 13
    run_and_check(cfg, weights, model, reqs, sched, dtype, "odd sizes")


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
    # too few pages for all at once: requests wait, or are preempted and recomputed (their states start again)
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
    folder = u.write_model(str(tmp_path_factory.mktemp("besulix_cli")), u.CFG_MAIN, weights)
    prompt = u.random_tokens(u.CFG_MAIN["vocab"], 9, 77)
    want = plain_greedy(u.CFG_MAIN, weights, prompt, 6)
    out = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "ferrox-amd"), "-m", folder, "--tokens",
                          ",".join(map(str, prompt)), "-n", "6", "--temp", "0", "--repeat-penalty", "1.0", "--ignore-eos", "--dtype", "float32",
                          "--block-size", "16", "--num-pages", "16"],
                         capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    assert ",".join(map(str, want)) in out.stdout.replace(" ", ""), (out.stdout[-500:], want)
    # random weights of the named shape, cut to two layers, through the command line
    out = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "ferrox-amd"), "--random-weights", "--config", "besulix-2k", "--layers", "2",
                          "--tokens", "1,2,3,4,5", "-n", "4", "--temp", "0", "--ignore-eos", "--num-pages", "8"],
                         capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    # the step-by-step replay: two requests, a portion beside a single token, logits at chosen places
    a, b = u.random_tokens(u.CFG_MAIN["vocab"], 30, 1), u.random_tokens(u.CFG_MAIN["vocab"], 4, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:17], "want": [0, 16]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[17:29], "want": []}, {"id": "b", "tokens": b[:3], "want": [2]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[3:], "want": [0]}, {"id": "a", "tokens": a[29:], "want": [0]}], "end": ["a", "b"]}]
    out_dir = str(tmp_path_factory.mktemp("besulix_replay"))
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
