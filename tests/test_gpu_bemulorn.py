"""Bemulorn on the GPU against the plain model (`plain_bemulorn`, NumPy float64): every kernel of its own
alone, each part alone in a one-layer model, then whole models of several tiny configurations under every
kind of schedule, in the 32-bit engine and in bfloat16 (held against the plain model with bfloat16
storage as a yardstick)."""

import copy
import io
import json

import numpy as np
import pytest
import torch

import plain_bemulorn as pb
import replay_util as ru
import tiny_bemulorn as tb

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = ["float32", "bfloat16"]
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def dev(values, dtype=torch.float32):
    return torch.from_numpy(np.ascontiguousarray(values)).to(device=DEV, dtype=dtype)


def ints(values):
    return torch.tensor([int(v) for v in values], dtype=torch.int32, device=DEV)


def rounded(values, dtype):
    """What the engine reads when `values` are stored in `dtype`, as float64."""
    return values.astype(np.float64) if dtype == "float32" else tb.bf16_round(values).astype(np.float64)


def tolerance(dtype, scale=1.0):
    return (2e-6 if dtype == "float32" else 1.2e-2) * scale


_ORACLES: dict = {}


def oracle(name, cfg, weights, tokens) -> ru.Oracle:
    key = (name, tuple(tokens))
    if key not in _ORACLES:
        wide = {k: v.astype(np.float64) for k, v in weights.items()}
        exact = pb.logits(cfg, wide, tokens)
        _ORACLES[key] = ru.Oracle(exact, pb.logits(cfg, wide, tokens, store=pb.bf16_round))
        # how far float32 storage and float32 rotation angles alone move the logits of this very input
        pb.ANGLE_TYPE = np.float32
        try:
            as_float32 = pb.logits(cfg, wide, tokens, store=pb.f32_round)
        finally:
            pb.ANGLE_TYPE = np.float64
        _ORACLES[key].moved_by_float32 = float(np.abs(as_float32 - exact).max())
    return _ORACLES[key]


def assert_close(got, want: ru.Oracle, dtype, what, bf16_max_factor=ru.BF16_MAX_FACTOR):
    """The engine against the plain model: bfloat16 against its yardstick; float32 within 1e-4, or, where
    float32 storage and angles alone move this input's logits further than half of that, within twice that far."""
    ru.assert_close(got, want, dtype, what, fp32_tol=max(ru.FP32_TOL, 2.0 * getattr(want, "moved_by_float32", 0.0)),
                    bf16_max_factor=bf16_max_factor)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    """Per configuration and engine dtype: (name of the pair, config, page size, weights, folder).  The
    bfloat16 engine gets weights whose experts are chosen steadily (see `tiny_bemulorn.make_weights`)."""
    out = {}
    for number, (name, (cfg, block)) in enumerate(tb.CONFIGS.items()):
        for dtype in DTYPES:
            weights = tb.make_weights(cfg, seed=70 + number, steady_choice=dtype == "bfloat16")
            folder = tb.write_model_dir(tmp_path_factory.mktemp("bemulorn") / f"{name}-{dtype}", cfg, weights)
            out[name, dtype] = (f"{name}-{dtype}", cfg, block, weights, folder)
    return out


def runner_for(folder, dtype, block, pages=64, seats=4, graphs=True):
    from mini_infer_amd.engine import ModelRunner

    return ModelRunner.from_pretrained(folder, dtype=dtype, num_blocks=pages, block_size=block, max_concurrent=seats,
                                       cuda_graph=graphs)


# ---------------------------------------------------------------------------------------------
# each kernel alone
# ---------------------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [10, 64, 2500])
def test_scaled_token_rows_plus_rows_by_position(dtype, width):
    from mini_infer_amd import ops

    rng = np.random.default_rng(width)
    table, rows = rng.standard_normal((31, width)).astype(np.float32), rng.standard_normal((40, width)).astype(np.float32)
    ids, positions = rng.integers(0, 31, 17), np.concatenate([[0, 39], rng.integers(0, 40, 15)])
    got = ops.embed_gather(dev(table, TORCH[dtype]), ints(ids), 2.7, dev(rows, TORCH[dtype]), ints(positions)).cpu().numpy()
    np.testing.assert_allclose(got, rounded(table, dtype)[ids] * 2.7 + rounded(rows, dtype)[positions], rtol=0, atol=2e-6)
    plain = ops.embed_gather(dev(table, TORCH[dtype]), ints(ids), 2.7).cpu().numpy()
    np.testing.assert_allclose(plain, rounded(table, dtype)[ids] * 2.7, rtol=0, atol=2e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 9, 40])
def test_logits_times_a_number(dtype, rows):
    from mini_infer_amd import ops

    rng = np.random.default_rng(rows)
    h, w = rng.standard_normal((rows, 64)).astype(np.float32), rng.standard_normal((90, 64)).astype(np.float32)
    scaled = ops.linear_f32_out(dev(h, TORCH[dtype]), dev(w, TORCH[dtype]), 1.75).cpu().numpy()
    plain = ops.linear_f32_out(dev(h, TORCH[dtype]), dev(w, TORCH[dtype])).cpu().numpy()
    np.testing.assert_array_equal(scaled, plain * np.float32(1.75))
    one_launch = ops.linear_f32_out(dev(h, TORCH[dtype]), dev(w, TORCH[dtype]), 1.75, dev(np.array([1.75], dtype=np.float32)))
    assert one_launch.dtype == torch.float32
    np.testing.assert_array_equal(one_launch.cpu().numpy(), scaled)
    np.testing.assert_allclose(plain, rounded(h, dtype) @ rounded(w, dtype).T, rtol=0, atol=tolerance(dtype, 30))


def pages_of(rows: np.ndarray, page_size: int, order: list[int], dtype, transposed=False) -> torch.Tensor:
    """[tokens, heads, dim] laid into pages, page i of the request at page id order[i]."""
    tokens, heads, dim = rows.shape
    pages = np.zeros((max(order) + 1, heads, page_size, dim), dtype=np.float32)
    for t in range(tokens):
        pages[order[t // page_size], :, t % page_size] = rows[t]
    made = dev(pages, TORCH[dtype])
    return made.transpose(2, 3).contiguous() if transposed else made


ROPE_CASES = [(4, 2, 16, 24, 12, 8, False), (3, 3, 10, 6, 6, 4, False), (8, 2, 64, 112, 32, 16, True), (4, 1, 96, 48, 96, 16, True),
              (2, 1, 8, 8, 0, 8, False), (5, 1, 32, 16, 8, 16, False)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("q_heads, kv_heads, dim, vdim, rot, page, transposed", ROPE_CASES)
def test_biases_partial_rotation_and_the_cache_write(dtype, q_heads, kv_heads, dim, vdim, rot, page, transposed):
    """Rows wider than q | k | v, scattered slots with a row that writes nothing, then a run of tokens that fills
    whole pages in order, and a layer that only rotates queries."""
    from mini_infer_amd import ops

    if transposed and dtype == "float32":
        pytest.skip("values lie transposed in the bfloat16 engine only")
    rng = np.random.default_rng(dim + rot)
    tokens = 2 * page + 5
    qw, kw, vw = q_heads * dim, kv_heads * dim, kv_heads * vdim
    rows = rng.standard_normal((tokens, qw + kw + vw + 16)).astype(np.float32) * 2
    bias = rng.standard_normal(qw + kw + vw).astype(np.float32)
    positions = rng.integers(0, 300, tokens)
    scale = {"base": 500.0, "dims": rot, "scaling": {"factor": 4.0, "original": 50, "fast": 6.0, "slow": 1.0}}
    turns, amplitude = pb.frequencies(scale) if rot else ([], 1.0)
    cos, sin = (torch.empty((tokens, 0), device=DEV),) * 2
    if rot:
        cos, sin = ops.rope_table(ints(positions), dev(np.array(turns, dtype=np.float32)), amplitude)
        angles = positions[:, None] * np.array(turns, dtype=np.float32).astype(np.float64)
        np.testing.assert_allclose(cos.cpu().numpy(), np.cos(angles) * amplitude, rtol=0, atol=1e-4)
    in_order = np.concatenate([np.arange(3 * page, 5 * page), [7, -1, 9, 10, 11][:5]])
    scattered = rng.permutation(5 * page)[:tokens]
    scattered[3] = -1
    r = rounded(rows, dtype)
    biased = r[:, : qw + kw + vw] + bias
    c, s = cos.double().cpu().numpy()[:, None, :], sin.double().cpu().numpy()[:, None, :]

    def turned(heads):
        out = heads.copy()
        half = rot // 2
        if half:
            out[..., :half] = heads[..., :half] * c - heads[..., half:rot] * s
            out[..., half:rot] = heads[..., half:rot] * c + heads[..., :half] * s
        return out

    want_q = turned(biased[:, :qw].reshape(tokens, q_heads, dim)).reshape(tokens, qw)
    want_k = turned(biased[:, qw:qw + kw].reshape(tokens, kv_heads, dim))
    want_v = biased[:, qw + kw:].reshape(tokens, kv_heads, vdim)
    for slots in (in_order, scattered):
        k_pages = torch.zeros((5, kv_heads, page, dim), dtype=TORCH[dtype], device=DEV)
        v_pages = torch.zeros((5, kv_heads, vdim, page) if transposed else (5, kv_heads, page, vdim), dtype=TORCH[dtype], device=DEV)
        qkv = dev(rows, TORCH[dtype])
        ops.rope_kv_write(qkv, cos, sin, ints(slots), k_pages, v_pages, q_heads=q_heads, kv_heads=kv_heads, head_dim=dim, rotary_dim=rot,
                          v_transposed=transposed, v_head_dim=vdim, bias=dev(bias))
        got = qkv.double().cpu().numpy()
        np.testing.assert_allclose(got[:, :qw], want_q, rtol=0, atol=tolerance(dtype, 4))
        np.testing.assert_array_equal(got[:, qw:], r[:, qw:])  # k, v and what follows stay
        kp = k_pages.double().cpu().numpy()
        vp = (v_pages.transpose(2, 3) if transposed else v_pages).double().cpu().numpy()
        for t, slot in enumerate(slots):
            if slot >= 0:
                np.testing.assert_allclose(kp[slot // page, :, slot % page], want_k[t], rtol=0, atol=tolerance(dtype, 4))
                np.testing.assert_allclose(vp[slot // page, :, slot % page], want_v[t], rtol=0, atol=tolerance(dtype, 4))
        assert np.count_nonzero(kp) <= (tokens - 1) * kw and np.count_nonzero(vp) <= (tokens - 1) * vw
    alone = dev(rows, TORCH[dtype])
    ops.rope_kv_write(alone, cos, sin, None, None, None, q_heads=q_heads, kv_heads=0, head_dim=dim, rotary_dim=rot, v_head_dim=vdim,
                      bias=dev(bias[:qw]))
    np.testing.assert_allclose(alone.double().cpu().numpy()[:, :qw], want_q, rtol=0, atol=tolerance(dtype, 4))
    np.testing.assert_array_equal(alone.double().cpu().numpy()[:, qw:], r[:, qw:])


ATTENTION_CASES = [  # heads, kv heads, key width, value width, page, chunk
    (4, 2, 64, 112, 16, 150), (8, 1, 96, 48, 16, 64), (8, 2, 128, 64, 16, 100), (6, 3, 64, 80, 16, 16), (4, 4, 192, 128, 16, 77),
    (16, 2, 96, 128, 16, 333), (2, 1, 128, 16, 16, 90), (5, 1, 64, 64, 16, 48), (4, 2, 32, 32, 32, 64), (4, 2, 10, 6, 4, 37),
    (3, 3, 40, 24, 8, 100), (2, 2, 256, 256, 16, 128), (32, 1, 128, 96, 16, 200)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads, kv_heads, dim, vdim, page, chunk", ATTENTION_CASES)
def test_attention_in_chunks_with_a_sink_gates_and_values_of_their_own_width(dtype, heads, kv_heads, dim, vdim, page, chunk):
    """Requests of unequal length side by side in scattered pages, into rows wider than the result: a prompt's
    last portion, two tokens, single tokens alone and together, and the same step with boundaries known on the
    device only.  In every request the last query's first head singles out the FIRST key of its chunk
    and its last head the last key of the chunk before, which must not show; head 1's first query
    has scores so low that the one added to the denominator takes nearly all the weight."""
    from mini_infer_amd import ops

    transposed = ops.mfma_attention_supported(TORCH[dtype], dim, page, vdim)
    assert transposed == (dtype == "bfloat16" and dim in (32, 64, 96, 128, 192, 256) and (page == 16 or dim == vdim))
    rng = np.random.default_rng(dim + vdim)
    scale, group = 1.0 / np.sqrt(dim), heads // kv_heads
    lengths = {"portion": (333, 70), "pair": (201, 2), "single": (160, 1), "early": (5, 3), "ones": (chunk + 1, 1)}
    made, pools, tables = {}, 0, {}
    for name, (keys_n, queries_n) in lengths.items():
        k = rng.standard_normal((keys_n, kv_heads, dim)).astype(np.float32)
        k[:, :, 0] = 1.0
        v = rng.standard_normal((keys_n, kv_heads, vdim)).astype(np.float32)
        q = rng.standard_normal((queries_n, heads, dim)).astype(np.float32)
        last = keys_n - 1
        first = last // chunk * chunk
        q[-1, 0] = 9.0 * np.sqrt(dim) * k[first, 0] / np.sum(k[first, 0] ** 2)
        if first > 0:
            away = k[first - 1, (heads - 1) // group]
            q[-1, -1] = 9.0 * np.sqrt(dim) * away / np.sum(away ** 2)
        if heads > 1 and queries_n > 1:
            q[0, 1] = 0.0
            q[0, 1, 0] = -10.0 * np.sqrt(dim)  # (the keys' first entry is 1: every score is -10)
        count = -(-keys_n // page)
        tables[name] = [pools + int(i) for i in rng.permutation(count)]
        pools += count
        made[name] = (k, v, q, rng.standard_normal((queries_n, heads)).astype(np.float32) * 2)
    k_pages = torch.zeros((pools, kv_heads, page, dim), dtype=TORCH[dtype], device=DEV)
    v_pages = torch.zeros((pools, kv_heads, vdim, page) if transposed else (pools, kv_heads, page, vdim), dtype=TORCH[dtype], device=DEV)
    for name, (k, v, _, _) in made.items():
        own = tables[name]
        local = list(range(len(own)))
        k_pages[own] = pages_of(k, page, local, dtype)
        v_pages[own] = pages_of(v, page, local, dtype, transposed)

    def want_of(name):
        k, v, q, gate = (rounded(a, dtype) for a in made[name])
        out = np.zeros((q.shape[0], heads, vdim))
        for i in range(q.shape[0]):
            p = k.shape[0] - q.shape[0] + i
            lo = p // chunk * chunk
            for a in range(heads):
                e = np.exp(k[lo:p + 1, a // group] @ q[i, a] * scale)
                out[i, a] = e @ v[lo:p + 1, a // group] / (1 + e.sum()) / (1 + np.exp(-gate[i, a]))
                if i == q.shape[0] - 1 and a == 0 and heads > 1 and p > lo:
                    assert e[0] / (1 + e.sum()) > 0.5  # the chunk's first key is what the answer is made of
        return out.reshape(q.shape[0], -1)

    def run(names, on_device=False):
        tokens = sum(lengths[n][1] for n in names)
        cu, pos, req = [0], [], []
        width = max(len(tables[n]) for n in names)
        table = np.full((len(names), width), -1)
        for b, n in enumerate(names):
            keys_n, queries_n = lengths[n]
            cu.append(cu[-1] + queries_n)
            pos += range(keys_n - queries_n, keys_n)
            req += [b] * queries_n
            table[b, :len(tables[n])] = tables[n]
            first = (keys_n - queries_n) // chunk * chunk
            table[b, :first // page] = -1  # pages of chunks that have ended were given back
        wide = torch.full((tokens, heads * dim + heads + 8), 7.0, dtype=TORCH[dtype], device=DEV)
        wide[:, :heads * dim] = dev(np.concatenate([made[n][2].reshape(-1, heads * dim) for n in names]), TORCH[dtype])
        wide[:, heads * dim:heads * dim + heads] = dev(np.concatenate([made[n][3] for n in names]), TORCH[dtype])
        if wide.stride(0) % 8:
            wide = torch.cat([wide, wide.new_zeros((tokens, 8 - wide.stride(0) % 8))], dim=1)
        out = torch.full((tokens, heads * vdim + 8), 3.0, dtype=TORCH[dtype], device=DEV)
        result = ops.paged_attention(
            wide, k_pages, v_pages, torch.tensor(table, dtype=torch.int32, device=DEV), ints(req), ints(pos), ints(cu),
            None if on_device else cu, q_heads=heads, kv_heads=kv_heads, head_dim=dim, scale=scale, window=None,
            max_seq_len=max(lengths[n][0] for n in names), v_transposed=transposed, v_head_dim=vdim, sink_logit=0.0, chunk=chunk,
            gate=wide[:, heads * dim:heads * dim + heads], out=out[:, :heads * vdim])
        assert result.data_ptr() == out.data_ptr() and bool((out[:, heads * vdim:] == 3.0).all())
        want = np.concatenate([want_of(n) for n in names])
        np.testing.assert_allclose(result.float().cpu().numpy(), want, rtol=0, atol=tolerance(dtype, 5), err_msg=f"{names} {on_device}")

    for names in (["portion"], ["single"], ["ones", "single"], ["single", "ones", "portion", "pair", "early"], ["early"]):
        print(names, flush=True)
        run(names)
    run(["single", "portion", "early", "pair"], on_device=True)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 7, 16, 30, 70])
@pytest.mark.parametrize("width, ff", [(64, 40), (192, 320), (90, 26)])
def test_the_clamped_activation_without_biases(dtype, rows, width, ff):
    from mini_infer_amd import ops

    rng = np.random.default_rng(rows + ff)
    x = rng.standard_normal((rows, width)).astype(np.float32)
    w = (rng.standard_normal((2 * ff, width)) * 2.5 / np.sqrt(width)).astype(np.float32)
    limit, slope = 1.3, 1.702
    both = rounded(x, dtype) @ rounded(w, dtype).T
    both = pb.bf16_round(both) if dtype == "bfloat16" else both
    g, u = np.minimum(both[:, :ff], limit), np.clip(both[:, ff:], -limit, limit)
    want = g / (1 + np.exp(-slope * g)) * (u + 1)
    got = ops.linear_clamped_glu(dev(x, TORCH[dtype]), dev(w, TORCH[dtype]), None, limit, slope)
    np.testing.assert_allclose(got.float().cpu().numpy(), want, rtol=0, atol=tolerance(dtype, 4))
    out = torch.full((rows, ff + 8), 5.0, dtype=TORCH[dtype], device=DEV)
    product = dev(both.astype(np.float32), TORCH[dtype])
    ops.clamped_glu(product, None, limit, slope, out=out[:, :ff])
    np.testing.assert_allclose(out[:, :ff].float().cpu().numpy(), want, rtol=0, atol=tolerance(dtype, 4))
    ops.gated_mul(product[:, :ff], product[:, ff:], "silu", out=out[:, :ff])
    z = rounded(both.astype(np.float32), dtype)
    np.testing.assert_allclose(out[:, :ff].float().cpu().numpy(), z[:, :ff] / (1 + np.exp(-z[:, :ff])) * z[:, ff:],
                               rtol=2e-6 if dtype == "float32" else 8e-3, atol=tolerance(dtype, 1))
    assert bool((out[:, ff:] == 5.0).all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows, width, outputs, top", [(1, 24, 3, 1), (9, 64, 6, 2), (40, 90, 5, 5), (33, 256, 16, 4), (8, 128, 200, 70), (300, 48, 7, 3)])
def test_the_router_by_the_softmax_over_the_chosen_logits(dtype, rows, width, outputs, top):
    """Biased logits are ranked (ties to the lower index) and weigh; the lists by expert hold every pair once."""
    from mini_infer_amd import ops

    rng = np.random.default_rng(rows * 3 + outputs)
    x = rng.standard_normal((rows, width)).astype(np.float32)
    router = (rng.standard_normal((outputs, width)) * 2.0 / np.sqrt(width)).astype(np.float32)
    bias = rng.standard_normal(outputs).astype(np.float32)
    if outputs > 4:
        router[2], bias[2] = router[1], bias[1]  # two experts no input tells apart
        bias[4] = -60.0  # one that nobody chooses (unless all are)
    z = rounded(x, dtype) @ router.astype(np.float64).T + bias
    picks = np.argsort(-z, axis=1, kind="stable")[:, :top]
    chosen_z = np.take_along_axis(z, picks, axis=1)
    share = np.exp(chosen_z - chosen_z[:, :1])
    share = share / share.sum(axis=1, keepdims=True) * 1.3
    xd = dev(x, TORCH[dtype])
    for experts in (None, outputs):
        chosen, weights, gates, *lists = ops.route_top_k(xd, dev(router), dev(bias), None, top=top, route_scale=1.3, scores="chosen_softmax",
                                                         experts=experts)
        assert gates is None
        close = np.abs(np.diff(np.sort(z, axis=1), axis=1)).min(axis=1) < 1e-5  # (rows whose order float32 sums may turn)
        tied = close & (outputs > 4)
        got = chosen.cpu().numpy()
        np.testing.assert_array_equal(got[~close], picks[~close])
        if tied.any():  # equal logits are bit-equal sums: the lower index stands first
            for row in got[tied]:
                where = {int(e): n for n, e in enumerate(row)}
                assert 2 not in where or (1 in where and where[1] < where[2])
        np.testing.assert_allclose(weights.cpu().numpy(), share, rtol=0, atol=3e-6)
        if experts is not None:
            listed, first = lists[0].listed.cpu().numpy(), lists[0].first.cpu().numpy()
            assert sorted(listed.tolist()) == list(range(rows * top)) and first[-1] == rows * top
            for e in range(outputs):
                assert all(got.reshape(-1)[p] == e for p in listed[first[e]:first[e + 1]])
    without, weights, _ = ops.route_top_k(xd, dev(router), None, None, top=top, route_scale=1.0, scores="chosen_softmax")
    np.testing.assert_allclose(weights.sum(dim=1).cpu().numpy(), 1.0, rtol=0, atol=3e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows, width, ff, experts, top", [(5, 64, 48, 6, 2), (70, 256, 128, 8, 3), (9, 90, 26, 3, 3)])
def test_experts_beside_a_shared_expert_without_a_gate_and_rows_left_for_the_norm(dtype, rows, width, ff, experts, top):
    from mini_infer_amd import ops

    rng = np.random.default_rng(width)
    x = rng.standard_normal((rows, width)).astype(np.float32)
    gate_up = (rng.standard_normal((experts, 2 * ff, width)) / np.sqrt(width)).astype(np.float32)
    down = (rng.standard_normal((experts, width, ff)) / np.sqrt(ff)).astype(np.float32)
    shared, other = (rng.standard_normal((rows, width)).astype(np.float32) for _ in range(2))
    stream, weight = rng.standard_normal((rows, width)).astype(np.float32), rng.uniform(0.5, 1.5, width).astype(np.float32)
    picks = np.stack([rng.permutation(experts)[:top] for _ in range(rows)])
    share = rng.uniform(0.1, 1.0, (rows, top)).astype(np.float32)
    xr, gr, dr = rounded(x, dtype), rounded(gate_up, dtype), rounded(down, dtype)
    routed = np.zeros((rows, width))
    for t in range(rows):
        for n, e in enumerate(picks[t]):
            g, u = gr[e, :ff] @ xr[t], gr[e, ff:] @ xr[t]
            routed[t] += share[t, n] * (dr[e] @ (g / (1 + np.exp(-g)) * u))
    args = (dev(x, TORCH[dtype]), dev(gate_up, TORCH[dtype]), dev(down, TORCH[dtype]), torch.tensor(picks, dtype=torch.int32, device=DEV), dev(share))
    sd = dev(shared, TORCH[dtype])
    forms = [ops.experts_few_rows, ops.experts_grouped]
    by_expert = ops.experts_by_expert_take(args[0], args[1])
    if by_expert:
        forms.append(ops.experts_by_expert)
    for form in forms:
        got = form(*args, sd, None).float().cpu().numpy()
        np.testing.assert_allclose(got, routed + rounded(shared, dtype), rtol=0, atol=tolerance(dtype, 10))
    if not by_expert:
        return
    apart = ops.experts_by_expert(*args, combine=False)
    assert isinstance(apart, ops.WeightedRows)
    np.testing.assert_allclose(apart.finish().float().cpu().numpy(), routed, rtol=0, atol=tolerance(dtype, 10))
    total = stream + rounded(other, dtype) + routed
    for listed in (None, [rows - 1, 0]):
        residual = dev(stream)
        got = ops.stream_update_norm(ops.StreamUpdate(dev(other, TORCH[dtype]), apart), residual, dev(weight, TORCH[dtype]), 1e-5,
                                     None if listed is None else ints(listed)).float().cpu().numpy()
        kept = total if listed is None else stream
        np.testing.assert_allclose(residual.cpu().numpy(), kept, rtol=0, atol=tolerance(dtype, 10))
        wanted = total if listed is None else total[listed]
        want = wanted / np.sqrt((wanted ** 2).mean(axis=1, keepdims=True) + 1e-5) * rounded(weight, dtype)
        np.testing.assert_allclose(got, want, rtol=0, atol=tolerance(dtype, 10))
    wide = dev(stream)
    wide += ops.StreamUpdate(dev(other, TORCH[dtype]), apart).finish()
    np.testing.assert_allclose(wide.cpu().numpy(), total, rtol=0, atol=tolerance(dtype, 10))


LAYER_IN_CASES = [  # q heads, kv heads, key width, value width, rotated dims, gate rows, ff, limit, hidden
    (8, 2, 64, 112, 32, 8, 320, 1.2, 192), (4, 1, 96, 48, 96, 8, 128, 0.0, 256), (12, 0, 64, 112, 32, 16, 0, 0.0, 192),
    (4, 4, 32, 32, 16, 8, 192, 1.2, 128), (3, 3, 8, 16, 0, 0, 4, 2.0, 64), (32, 8, 128, 128, 64, 32, 1024, 7.0, 1024), (1, 1, 128, 128, 128, 8, 8, 1.0, 96)]


@pytest.mark.parametrize("rows", [1, 5, 16, 27, 32])
@pytest.mark.parametrize("case", range(len(LAYER_IN_CASES)))
def test_a_layers_first_product_with_all_that_follows_folded_in(rows, case):
    """One kernel against the product, the biased rotation with its cache write and the activation in turn, on
    plain rows and (up to 16) on rows whose norm factors are apart."""
    from mini_infer_amd import ops

    q_heads, kv_heads, dim, vdim, rot, gate_rows, ff, limit, hidden = LAYER_IN_CASES[case]
    layout = ops.LayerInputs(q_heads, kv_heads, dim, vdim, gate_rows, ff, limit, 1.702)
    rng = np.random.default_rng(case * 100 + rows)
    page, pages = 16, 5
    bf = torch.bfloat16
    x = dev(rng.standard_normal((rows, hidden)).astype(np.float32), bf)
    total = -(-layout.rows // 8) * 8
    w_np = (rng.standard_normal((total, hidden)) * 1.5 / np.sqrt(hidden)).astype(np.float32)
    w_np[layout.qkv_rows + q_heads: layout.qkv_rows + gate_rows] = 0.0
    w = dev(w_np, bf)
    bias = dev(rng.standard_normal(layout.qkv_rows).astype(np.float32))
    cos = sin = torch.empty((rows, 0), device=DEV)
    if rot:
        cos, sin = ops.rope_table(ints(rng.integers(0, 500, rows)), dev((1000.0 ** (-np.arange(rot // 2) / (rot // 2))).astype(np.float32)), 1.2)
    transposed = vdim != 16
    slots = rng.permutation(pages * page)[:rows]
    if rows > 3:
        slots[2] = -1

    def new_pages():
        k = torch.zeros((pages, max(kv_heads, 1), page, dim), dtype=bf, device=DEV)
        return k, torch.zeros((pages, max(kv_heads, 1), vdim, page) if transposed else (pages, max(kv_heads, 1), page, vdim), dtype=bf, device=DEV)

    def in_turn(product):
        k, v = new_pages()
        product = product.clone()
        ops.rope_kv_write(product, cos, sin, ints(slots) if kv_heads else None, k, v, q_heads=q_heads, kv_heads=kv_heads, head_dim=dim,
                          rotary_dim=rot, v_transposed=transposed, v_head_dim=vdim, bias=bias)
        act = None
        if ff:
            cols = product[:, layout.qkv_rows + gate_rows: layout.rows]
            act = ops.clamped_glu(cols, None, limit, 1.702) if limit else ops.gated_mul(cols[:, :ff], cols[:, ff:], "silu")
        gates = product[:, layout.qkv_rows: layout.qkv_rows + q_heads] if gate_rows else None
        return product[:, : q_heads * dim], gates, act, k, v

    inputs = [(x, ops.linear(x, w) if rows <= 16 else None)]
    if rows <= 16:
        sumsq = dev(rng.uniform(0.2, 0.6, (3, rows)).astype(np.float32) * hidden / 3)
        factor = torch.rsqrt(sumsq.sum(dim=0) / hidden + 1e-5)
        exact = (x.double() @ w.double().t()) * factor.double()[:, None]
        inputs.append((ops.ScaledRows(x, sumsq, 1e-5), exact.to(bf)))
    for source, product in inputs:
        exact_bits = product is not None and not isinstance(source, ops.ScaledRows)
        if product is None:
            product = torch.matmul(x, w.t())
        want = in_turn(product)
        k, v = new_pages()
        holder = torch.full((rows, ff + 16), 9.0, dtype=bf, device=DEV)
        queries, gates = ops.layer_in(source, w, layout, cos, sin, rot, ints(slots) if kv_heads else None, k, v, v_transposed=transposed,
                                      bias=bias, activated=holder[:, :ff] if ff else None)
        got = (queries, gates, holder[:, :ff] if ff else None, k, v)
        for name, a, b in zip(("queries", "gates", "activation", "keys", "values"), got, want):
            assert (a is None) == (b is None), name
            if a is None:
                continue
            if exact_bits and name in ("gates", "values"):  # (what is rotated or activated may differ in how a multiply-add is contracted)
                assert torch.equal(a, b), name
            else:
                np.testing.assert_allclose(a.float().cpu().numpy(), b.float().cpu().numpy(), rtol=1.6e-2, atol=2e-2, err_msg=name)
        assert bool((holder[:, ff:] == 9.0).all())
        if kv_heads == 0:
            assert not k.any() and not v.any()


# ---------------------------------------------------------------------------------------------
# each part alone in a one-layer model
# ---------------------------------------------------------------------------------------------

ALONE = {
    "attention": tb.attention(4, 2, 16, 24, 0.5, chunk=13, rot=tb.YARN_A),
    "attention_plain": tb.attention(3, 3, 10, 6, 0.7),
    "attention_folded": tb.attention(4, 2, 64, 80, 0.2, chunk=20, rot=tb.YARN_C),
    "experts": tb.attention(2, 2, 8, 8, 0.6, chunk=9, mlp=tb.moe(24, 5, 3, shared=20)),
    "experts_alone": tb.attention(2, 1, 8, 8, 0.6, chunk=30, mlp=tb.moe(32, 4, 1)),
    "dense": tb.attention(2, 1, 8, 16, 0.6, chunk=2, rot=tb.rotation(30.0, 8), mlp=tb.dense(48, 0.9)),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("part", sorted(ALONE))
def test_each_part_alone_whole_and_token_by_token(tmp_path, dtype, part):
    from mini_infer_amd.engine import StepEntry

    cfg = tb.config(90, 64, [ALONE[part]], eps=1e-5, scale=1.3, logit_scale=0.9, positions=60)
    weights = tb.make_weights(cfg, seed=len(part), steady_choice=dtype == "bfloat16")
    folder = tb.write_model_dir(tmp_path / "m", cfg, weights)
    tokens = tb.random_tokens(cfg, 45, seed=9)
    want = oracle(f"{part}-{dtype}", cfg, weights, tokens)
    runner = runner_for(folder, dtype, 16, pages=8, seats=2)
    whole = runner.step([StepEntry("w", tokens, list(range(45)))]).cpu().numpy()
    # (one layer, 45 tokens: the yardstick's largest error is the largest of few draws, so it gets more room)
    assert_close(whole, want, dtype, f"{part} whole", bf16_max_factor=3.0)
    one_by_one = np.concatenate([runner.step([StepEntry("d", [t], [0])]).cpu().numpy() for t in tokens])
    assert_close(one_by_one, want, dtype, f"{part} token by token", bf16_max_factor=3.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "C", "E"])
def test_products_made_together_and_apart_agree(folders, dtype, name):
    """The same weights in blocks whose sublayers make their products on their own: a prompt, a portion of
    two tokens and decoded ones, in steps launched kernel by kernel and recorded."""
    from mini_infer_amd.engine import ModelRunner, StepEntry
    from mini_infer_amd.models import architecture_for
    from mini_infer_amd.models.decoder import DecoderModel
    from mini_infer_amd.weights import load_checkpoint

    name, cfg, block, weights, folder = folders[name, dtype]
    arch = architecture_for(cfg)
    spec = arch.build_spec(arch.parse_config(cfg))
    for layer in spec.layers:
        layer.block["joint"] = False
    model = DecoderModel(spec, TORCH[dtype], torch.device(DEV))
    load_checkpoint(model, folder)
    assert all(b.joint is None for b in model.blocks)
    tokens = tb.random_tokens(cfg, 60, seed=17)
    portions = [tokens[:40], tokens[40:42]] + [[t] for t in tokens[42:]]
    want = oracle(name, cfg, weights, tokens)
    for graphs in (True, False):
        for runner in (ModelRunner(model, None, num_blocks=8, block_size=block, max_concurrent=1, cuda_graph=graphs),
                       runner_for(folder, dtype, block, pages=8, seats=1, graphs=graphs)):
            got = np.concatenate([runner.step([StepEntry("a", part, list(range(len(part))))]).cpu().numpy() for part in portions])
            assert_close(got, want, dtype, f"{name} graphs={graphs}", bf16_max_factor=2.5)


@pytest.mark.parametrize("name", ["A", "C", "E"])
def test_a_prompts_products_made_in_their_two_parts_agree_too(folders, name, monkeypatch):
    """What very large products of many rows do, with limits so low that the tiny ones do it: the parts' own views of
    the stacked matrices, in whole prompts, portions and decoded tokens."""
    from mini_infer_amd.engine import StepEntry
    from mini_infer_amd.parts import joint

    name, cfg, block, weights, folder = folders[name, "bfloat16"]
    tokens = tb.random_tokens(cfg, 60, seed=17)
    want = oracle(name, cfg, weights, tokens)
    made = {"out": 0}
    original = joint.JointProducts.outputs

    def counted(self, joined):
        made["out"] += 1
        return original(self, joined)

    monkeypatch.setattr(joint.JointProducts, "outputs", counted)
    for rows, outputs in ((2, 1), (0, 1), (2, 1 << 40)):
        monkeypatch.setattr(joint, "APART_IN_OUTPUTS", outputs)
        monkeypatch.setattr(joint, "APART_OUT_ROWS", rows)
        monkeypatch.setattr(joint, "APART_OUT_K", 0)
        before = made["out"]
        runner = runner_for(folder, "bfloat16", block, pages=8, seats=1, graphs=False)
        portions = [tokens[:40], tokens[40:42]] + [[t] for t in tokens[42:]]
        got = np.concatenate([runner.step([StepEntry("a", part, list(range(len(part))))]).cpu().numpy() for part in portions])
        assert_close(got, want, "bfloat16", f"{name} {rows} {outputs}", bf16_max_factor=2.5)
        assert made["out"] > before


def test_a_step_past_the_table_of_positions_is_refused_and_changes_nothing(tmp_path):
    from mini_infer_amd.engine import StepEntry
    from mini_infer_amd.engine.llm import LLM

    cfg = tb.config(60, 64, [tb.attention(2, 1, 16, 16, 0.4, chunk=12, mlp=tb.dense(32, 2.0))], eps=1e-5, positions=30)
    weights = tb.make_weights(cfg, seed=1)
    folder = tb.write_model_dir(tmp_path / "m", cfg, weights)
    tokens = tb.random_tokens(cfg, 31, seed=2)
    runner = runner_for(folder, "float32", 8, pages=8, seats=2)
    with pytest.raises(ValueError, match="positions"):
        runner.step([StepEntry("a", tokens, [30])])
    assert not runner.has_request("a")
    got = runner.step([StepEntry("a", tokens[:29], list(range(29)))]).cpu().numpy()
    with pytest.raises(ValueError, match="positions"):
        runner.step([StepEntry("a", tokens[29:31], [1])])
    got = np.concatenate([got, runner.step([StepEntry("a", tokens[29:30], [0])]).cpu().numpy()])
    wide = {k: v.astype(np.float64) for k, v in weights.items()}
    np.testing.assert_allclose(got, pb.logits(cfg, wide, tokens[:30]), rtol=0, atol=ru.FP32_TOL)
    with pytest.raises(ValueError, match="positions"):
        runner.step([StepEntry("a", tokens[30:], [0])])
    # the scheduler rejects what cannot fit and serves what just does
    llm = LLM(folder, dtype="float32", num_blocks=8, block_size=8, max_concurrent=2)
    fits, too_long = llm.generate([tokens[:21], tokens[:22]], max_tokens=10)  # (the last token is never fed)
    assert len(fits.tokens) == 10 and fits.finish_reason == "length" and too_long.finish_reason == "cancelled" and not too_long.tokens


# ---------------------------------------------------------------------------------------------
# whole models under every kind of schedule
# ---------------------------------------------------------------------------------------------

LENGTHS = {"A": (70, 41, 9, 33, 58, 1), "B": (45, 64, 17, 2, 39), "C": (130, 40, 77, 5), "D": (50, 21, 36, 3, 44), "E": (110, 97, 4, 62)}


def requests_of(name, cfg):
    return {f"{name}{i}": tb.random_tokens(cfg, n, seed=100 * len(name) + 7 * i + n) for i, n in enumerate(LENGTHS[name])}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(tb.CONFIGS))
@pytest.mark.parametrize("family", ["whole", "decode", "portions", "mixed"])
def test_logits_do_not_depend_on_the_schedule(folders, name, dtype, family):
    """Whole prompts; a prompt and then its last tokens one by one (chunks begin and end among decoded
    tokens); portions down to two tokens; up to four live requests of unequal length in one batch, in
    a pool so small that pages and seats are used again.  Each request is held against itself alone."""
    name, cfg, block, weights, folder = folders[name, dtype]
    requests = requests_of(name[0], cfg)
    schedule = {
        "whole": lambda: ru.schedule_whole(requests),
        "decode": lambda: ru.schedule_prefill_then_decode(requests, tail=36),
        "portions": lambda: ru.schedule_portions(requests, seed=3),
        "mixed": lambda: ru.schedule_mixed(requests, seed=5, max_live=4, tail=12),
    }[family]()
    pages = ru.peak_pages(requests, schedule, block)
    runner = runner_for(folder, dtype, block, pages=pages, seats=4 if family == "mixed" else 1)
    got = ru.run_schedule(runner, requests, schedule)
    for rid, tokens in requests.items():
        assert_close(got[rid], oracle(name, cfg, weights, tokens), dtype, f"{name} {family} {rid}")
    runner.cache.check()
    assert runner.cache.states.num_free == runner.cache.states.max_requests
    assert runner.num_free_blocks() == pages


def test_the_stream_after_every_layer(folders):
    """The 32-bit engine's float32 stream where a layer's sum has been added to it, against the plain model's."""
    from mini_infer_amd.engine import StepEntry
    from mini_infer_amd.parts.norm import RMSNorm

    name, cfg, block, weights, folder = folders["A", "float32"]
    tokens = tb.random_tokens(cfg, 37, seed=5)
    seen = []
    original = RMSNorm.forward

    def watching(self, delta, residual, rows=None):
        if rows is not None:  # (the final norm leaves the stream as it is: add what is pending here)
            seen.append((residual + (delta.finish() if hasattr(delta, "finish") else delta)).cpu().numpy())
        out = original(self, delta, residual, rows)
        if rows is None and delta is not None:
            seen.append(residual.cpu().numpy())
        return out

    runner = runner_for(folder, "float32", block, pages=8, seats=1, graphs=False)
    RMSNorm.forward = watching
    try:
        runner.step([StepEntry("a", tokens, [36])])
    finally:
        RMSNorm.forward = original
    layers = []
    pb.logits(cfg, {k: v.astype(np.float64) for k, v in weights.items()}, tokens, layers_out=layers)
    assert len(seen) == len(layers) == len(cfg["layers"])
    for n, (a, b) in enumerate(zip(seen, layers)):
        np.testing.assert_allclose(a, b, rtol=0, atol=5e-5, err_msg=f"layer {n}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_pages_and_seats_used_again_start_clean(folders, dtype):
    from mini_infer_amd.engine import StepEntry

    name, cfg, block, weights, folder = folders["A", dtype]
    first, second = tb.random_tokens(cfg, 30, seed=1), tb.random_tokens(cfg, 26, seed=2)
    runner = runner_for(folder, dtype, block, pages=2, seats=1)
    runner.step([StepEntry("a", first, [])])
    slot = runner.cache.state_slot("a")
    runner.free_request("a")
    got = runner.step([StepEntry("b", second[:2], [0, 1])]).cpu().numpy()
    assert runner.cache.state_slot("b") == slot
    got = np.concatenate([got, runner.step([StepEntry("b", second[2:], list(range(24)))]).cpu().numpy()])
    assert_close(got, oracle(name, cfg, weights, second), dtype, "second owner of pages and seat")


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_failing_step_leaves_no_trace(folders, dtype, monkeypatch):
    from mini_infer_amd.engine import StepEntry

    name, cfg, block, weights, folder = folders["A", dtype]
    tokens = tb.random_tokens(cfg, 40, seed=8)
    runner = runner_for(folder, dtype, block, pages=4, seats=1, graphs=False)
    got = [runner.step([StepEntry("a", tokens[:11], list(range(11)))]).cpu().numpy()]

    def refuse(*args, **kwargs):
        raise RuntimeError("refused")

    for part in (tokens[11:13], tokens[13:14], tokens[14:40]):
        monkeypatch.setattr(runner.model.head, "forward", refuse)
        with pytest.raises(RuntimeError, match="refused"):
            runner.step([StepEntry("a", part, [0])])
        monkeypatch.undo()
        got.append(runner.step([StepEntry("a", part, list(range(len(part))))]).cpu().numpy())
    assert_close(np.concatenate(got), oracle(name, cfg, weights, tokens), dtype, "after refused steps")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "C", "E"])
def test_long_decoding_through_recorded_steps(folders, dtype, name):
    """Two requests decoded side by side for 150 steps after prompts of 130 and 7 tokens, across many page and
    chunk borders; the single-token steps are replayed graphs, with eager work between them."""
    from mini_infer_amd.engine import StepEntry

    name, cfg, block, weights, folder = folders[name, dtype]
    requests = {"x": tb.random_tokens(cfg, 280, seed=31), "y": tb.random_tokens(cfg, 157, seed=32)}
    runner = runner_for(folder, dtype, block, pages=34, seats=3)
    got = {rid: [] for rid in requests}
    both = runner.step([StepEntry("x", requests["x"][:130], list(range(130))), StepEntry("y", requests["y"][:7], list(range(7)))]).cpu().numpy()
    got["x"].append(both[:130])
    got["y"].append(both[130:])
    for k in range(150):
        if k in (20, 70):  # a prompt of another request between the replays
            runner.step([StepEntry("z", tb.random_tokens(cfg, 40, seed=k), [39])])
            runner.free_request("z")
        logits = runner.step([StepEntry("x", [requests["x"][130 + k]], [0]), StepEntry("y", [requests["y"][7 + k]], [0])]).cpu().numpy()
        got["x"].append(logits[:1])
        got["y"].append(logits[1:])
    assert runner.decode_graphs is not None and runner.decode_graphs.replays == 150
    for rid, tokens in requests.items():
        assert_close(np.concatenate(got[rid]), oracle(name, cfg, weights, tokens), dtype, f"long decoding {rid}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_request_outlives_the_pool_where_chunks_give_their_pages_back(folders, dtype):
    """Configuration E (chunks of 96 and 80, pages of 16): 250 positions in a pool of 8 pages, decoded and in
    portions; the longest chunk holds 6 of them and the one before it is given back when it ends."""
    from mini_infer_amd.engine import StepEntry

    name, cfg, block, weights, folder = folders["E", dtype]
    tokens = tb.random_tokens(cfg, 250, seed=91)
    want = oracle(name, cfg, weights, tokens)
    for portions in ([tokens[:90]] + [[t] for t in tokens[90:]], [tokens[i:i + 15] for i in range(0, 250, 15)]):
        runner = runner_for(folder, dtype, block, pages=8, seats=1)
        got = np.concatenate([runner.step([StepEntry("a", part, list(range(len(part))))]).cpu().numpy() for part in portions])
        assert_close(got, want, dtype, f"{len(portions)} portions")
        runner.cache.check()
        runner.free_request("a")
        assert runner.num_free_blocks() == 8


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("fast", [True, False])
def test_one_far_key_is_found_inside_its_chunk_and_not_beyond_it(tmp_path, dtype, fast):
    """Two layers, the second reading the first's keys with a chunk of its own, whose first head singles out one
    token far back: at the chunk's first position, at page borders, inside, and one before the chunk (which must
    not show).  The engine agrees with every sequence in a whole prompt, in portions and decoded."""
    from mini_infer_amd.engine import StepEntry

    sizes = (64, 80) if fast else (18, 10)
    chunk, length = 140, 276  # the last query's chunk is 140 .. 279
    layers = [tb.attention(4, 2, *sizes, 0.2, chunk=chunk), tb.attention(4, 2, *sizes, 0.2, chunk=chunk, mlp=tb.dense(32, 3.0), kv_from=0)]
    cfg = tb.config(60, 64, layers, eps=1e-5, positions=300)
    weights = tb.make_weights(cfg, seed=12)
    key_token, query_token = 58, 59
    weights["embed"][:, 1:3] = weights["pos"][:, 1:3] = 0.0
    weights["embed"][key_token, 1] = weights["embed"][query_token, 2] = 5.0
    weights["head"][:, 1:3] = 0.0
    for n in range(2):
        weights[f"l{n}.norm1"][1:3] = 1.0
        weights[f"l{n}.mix.o"][1:3] = 0.0
        weights[f"l{n}.mix.q"][0] = 0.0
        weights[f"l{n}.mix.q"][0, 2] = 4.0  # the first head's first query entry reads the query token alone
        weights[f"l{n}.mix.q.b"][0] = 0.0
        weights[f"l{n}.mix.g"][0] = 0.0  # (its gate stands at a half)
    weights["l0.mix.k"][0] = 0.0
    weights["l0.mix.k"][0, 1] = 4.0  # and its first key entry the key token alone
    weights["l0.mix.k.b"][0] = 0.0
    weights = {k: tb.bf16_round(v) for k, v in weights.items()}
    folder = tb.write_model_dir(tmp_path / "m", cfg, weights)
    base = [t % 58 for t in tb.random_tokens(cfg, length, seed=4)]
    base[-1] = query_token
    runner = runner_for(folder, dtype, 16, pages=20, seats=1)
    plain = oracle(f"far-{fast}-none", cfg, weights, base)
    for place in (0, 139, 140, 143, 144, 159, 160, 200, 255, 256, 274):
        tokens = list(base)
        tokens[place] = key_token
        want = oracle(f"far-{fast}-{place}", cfg, weights, tokens)
        shows = float(np.abs(want.exact[-1] - plain.exact[-1]).max())
        if place < chunk:
            assert shows == 0.0
        else:
            assert shows > 5 * max(plain.yard_p99, 0.01), f"key at {place}: {shows:.3f} against {plain.yard_p99:.3f}"
        runs = {"whole": [tokens], "portions": [tokens[:40], tokens[40:42], tokens[42:275], tokens[275:]],
                "decoded": [tokens[:271]] + [[t] for t in tokens[271:]]}
        for how, portions in runs.items():
            for part in portions:
                logits = runner.step([StepEntry(how, part, [len(part) - 1])]).cpu().numpy()
            runner.free_request(how)
            last = want[slice(length - 1, length)]
            last.moved_by_float32 = want.moved_by_float32
            assert_close(logits, last, dtype, f"{how}, key at {place}", bf16_max_factor=3.0)


def resized(cfg, layer, by):
    other = copy.deepcopy(cfg)
    other["layers"][layer]["mixer"] = {**other["layers"][layer]["mixer"], "mask": {"size": other["layers"][layer]["mixer"]["mask"]["size"] + by}}
    return other


def test_every_chunk_ends_where_it_should_beside_page_borders(folders):
    """Pages of 4 and chunks of 4, 5, 8, 3 and 1: the engine agrees with the plain model of these chunks, in a
    whole prompt, in portions of two and token by token, and is far from the plain models whose chunk in any one layer
    is a position longer or shorter."""
    from mini_infer_amd.engine import StepEntry

    _, cfg, block, weights, folder = folders["D", "float32"]
    tokens = tb.random_tokens(cfg, 40, seed=77)
    wide = {k: v.astype(np.float64) for k, v in weights.items()}
    want = pb.logits(cfg, wide, tokens)
    runner = runner_for(folder, "float32", block, pages=12, seats=1)
    runs = {
        "whole": [tokens],
        "pairs": [tokens[i:i + 2] for i in range(0, 40, 2)],
        "decoded": [tokens[:3]] + [[t] for t in tokens[3:]],
    }
    for how, portions in runs.items():
        got = np.concatenate([runner.step([StepEntry(how, part, list(range(len(part))))]).cpu().numpy() for part in portions])
        runner.free_request(how)
        assert np.abs(got - want).max() < ru.FP32_TOL, how
        for layer in range(len(cfg["layers"])):
            for by in (-1, 1):
                if cfg["layers"][layer]["mixer"]["mask"]["size"] + by < 1:
                    continue
                other = pb.logits(resized(cfg, layer, by), wide, tokens)
                assert np.abs(other - want).max() > 100 * ru.FP32_TOL  # the test can tell
                assert np.abs(got - other).max() > 100 * ru.FP32_TOL, f"{how}: chunk of layer {layer} off by {by}"


@pytest.mark.parametrize("name", ["A", "B"])
def test_greedy_generation_through_llm_and_the_scheduler(folders, name):
    """Five prompts for two seats, prompts cut into portions of 8 under a 20-token budget: every generated
    token is the plain model's greedy choice."""
    from mini_infer_amd.engine.llm import LLM

    _, cfg, block, weights, folder = folders[name, "float32"]
    wide = {k: v.astype(np.float64) for k, v in weights.items()}
    lengths, new_tokens = (5, 19, 33, 2, 11), 9
    prompts = [tb.random_tokens(cfg, n, seed=300 + n) for n in lengths]
    llm = LLM(folder, dtype="float32", num_blocks=12, block_size=block, max_concurrent=2, max_num_batched_tokens=20, chunk_size=8)
    results = llm.generate(prompts, max_tokens=new_tokens)
    for prompt, result in zip(prompts, results):
        sequence = list(prompt)
        for _ in range(new_tokens):
            sequence.append(pb.greedy(pb.logits(cfg, wide, sequence)[-1]))
        assert result.tokens == sequence[len(prompt):] and result.finish_reason == "length"
    assert llm.runner.cache.states.num_free == 2
    llm.runner.cache.check()


def test_the_command_line_writes_random_weights_and_generates_greedily_and_by_seeded_sampling(tmp_path, capsys):
    """`random-weights` from a config.json, then `generate`: greedy twice the same, sampled with one seed
    twice the same and (at this temperature) different from greedy."""
    from mini_infer_amd.__main__ import main

    cfg, block = tb.CONFIGS["A"]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    assert main(["random-weights", "--config", str(tmp_path / "config.json"), "--seed", "3", "--out", str(tmp_path / "m"),
                 "--std", "0.3", "--norm-jitter", "0.1"]) == 0
    capsys.readouterr()

    def generate(*extra):
        assert main(["generate", "--model", str(tmp_path / "m"), "--prompt-ids", "5 9 100 3 77", "--prompt-ids", "1,2",
                     "--max-tokens", "12", "--num-blocks", "16", "--block-size", str(block), "--max-concurrent", "2",
                     "--ignore-eos", *extra]) == 0
        lines = [json.loads(line) for line in capsys.readouterr().out.strip().splitlines()]
        assert [line["prompt_tokens"] for line in lines] == [5, 2] and all(len(line["tokens"]) == 12 for line in lines)
        return [line["tokens"] for line in lines]

    greedy = generate()
    assert generate() == greedy
    sampled = generate("--temperature", "1.5", "--top-k", "40", "--top-p", "0.95", "--seed", "11")
    assert generate("--temperature", "1.5", "--top-k", "40", "--top-p", "0.95", "--seed", "11") == sampled
    assert sampled != greedy and all(0 <= t < cfg["vocab"] for tokens in sampled for t in tokens)


def test_the_replay_program_runs_a_trace_of_this_design(folders, tmp_path):
    from mini_infer_amd.engine import replay, trace

    name, cfg, block, weights, folder = folders["B", "float32"]
    requests = {f"t{i}": tb.random_tokens(cfg, n, seed=i) for i, n in enumerate((70, 41, 9, 33, 58))}
    schedule = trace.make_schedule("mixed", requests, seed=1, tail=10)
    lines = trace.to_trace_lines(requests, schedule)
    limit = trace.peak_pages(requests, schedule, 64) * 64
    args = replay.build_parser().parse_args(["--model", str(folder), "--dtype", "float32", "--out", str(tmp_path / "out"),
                                             "--max-tokens", str(limit)])
    said = io.StringIO()
    assert replay.run(args, lines=lines, out=said) == 0
    assert said.getvalue().split() == [w for n in range(len(lines)) for w in ("done", str(n))]
    fed = {rid: 0 for rid in requests}
    for number, line in enumerate(lines):
        step = json.loads(line)
        got = np.fromfile(tmp_path / "out" / f"{number}.f32", dtype="<f4").reshape(-1, cfg["vocab"])
        at = 0
        for entry in step["entries"]:
            n, rid = len(entry["tokens"]), entry["id"]
            whole = oracle(name, cfg, weights, requests[rid])
            want = whole[slice(fed[rid], fed[rid] + n)]
            want.moved_by_float32 = whole.moved_by_float32
            assert_close(got[at: at + n], want, "float32", f"trace step {number} {rid}")
            fed[rid] += n
            at += n
