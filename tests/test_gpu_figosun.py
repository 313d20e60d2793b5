"""Figosun on the GPU against the plain model (`plain_figosun`, NumPy float64): every kernel of its own
alone, each part alone in a one-layer model, then whole models of several tiny configurations under
every kind of schedule, in the 32-bit engine and in bfloat16 (held against the plain model with bfloat16
storage as a yardstick)."""

import io
import json

import numpy as np
import pytest
import torch

import plain_figosun as pf
import replay_util as ru
import tiny_figosun as tf

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = ["float32", "bfloat16"]
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def dev(values, dtype=torch.float32):
    return torch.from_numpy(np.ascontiguousarray(values)).to(device=DEV, dtype=dtype)


def ints(values):
    return torch.tensor(np.asarray(values).tolist(), dtype=torch.int32, device=DEV)


def rounded(values, dtype):
    """What the engine reads when `values` are stored in `dtype`, as float64."""
    return values.astype(np.float64) if dtype == "float32" else tf.bf16_round(values).astype(np.float64)


def tolerance(dtype, scale=1.0):
    return (2e-6 if dtype == "float32" else 1.2e-2) * scale


_ORACLES: dict = {}


def oracle(name, cfg, weights, tokens) -> ru.Oracle:
    key = (name, tuple(tokens))
    if key not in _ORACLES:
        wide = {k: v.astype(np.float64) for k, v in weights.items()}
        _ORACLES[key] = ru.Oracle(pf.logits(cfg, wide, tokens), pf.logits(cfg, wide, tokens, store=pf.bf16_round))
        pf.ANGLE_TYPE = np.float32
        try:  # how far float32 storage and angles alone, with exact arithmetic between, move the logits of this very input
            moved = float(np.abs(pf.logits(cfg, wide, tokens, store=pf.f32_round) - _ORACLES[key].exact).max())
        finally:
            pf.ANGLE_TYPE = np.float64
        _ORACLES[key].moved_by_float32 = moved
    return _ORACLES[key]


def assert_close(got, want: ru.Oracle, dtype, what, bf16_max_factor=ru.BF16_MAX_FACTOR):
    """The engine against the plain model: bfloat16 against its yardstick; float32 within 1e-4, or, where
    float32 storage and angles alone move this input's logits further than half of that, within twice that far."""
    ru.assert_close(got, want, dtype, what, fp32_tol=max(ru.FP32_TOL, 2.0 * getattr(want, "moved_by_float32", 0.0)),
                    bf16_max_factor=bf16_max_factor)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    """Per configuration and engine dtype: (name of the pair, config, page size, weights, folder).  The bfloat16
    engine gets weights whose experts are chosen steadily (see `tiny_figosun.make_weights`)."""
    out = {}
    for number, (name, (cfg, block)) in enumerate(tf.CONFIGS.items()):
        for dtype in DTYPES:
            weights = tf.make_weights(cfg, seed=70 + number, steady_choice=dtype == "bfloat16")
            folder = tf.write_model_dir(tmp_path_factory.mktemp("figosun") / f"{name}-{dtype}", cfg, weights)
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
@pytest.mark.parametrize("width", [10, 64, 2500, 5001])
@pytest.mark.parametrize("pieces, gated", [(1, True), (3, True), (2, False)])
def test_gated_update_and_both_norms(dtype, width, pieces, gated):
    from mini_infer_amd import ops

    rng = np.random.default_rng(width + pieces)
    rows, eps_out, eps = 7, 1e-3, 1e-5
    x = rng.standard_normal((rows, width)).astype(np.float32) * 2
    y = rng.standard_normal((rows * pieces, width)).astype(np.float32)
    gate = rng.standard_normal((rows, width + 4)).astype(np.float32) * 2
    bias = rng.standard_normal(width).astype(np.float32)
    w_out, w = (rng.uniform(0.5, 1.5, width).astype(np.float32) for _ in range(2))
    v = rounded(y, dtype).reshape(rows, pieces, width).sum(axis=1)
    if gated:
        v = v / (1 + np.exp(-(rounded(gate, dtype)[:, :width] + bias)))
    after = x + v / np.sqrt((v ** 2).mean(axis=1, keepdims=True) + eps_out) * rounded(w_out, dtype)
    normed = after / np.sqrt((after ** 2).mean(axis=1, keepdims=True) + eps) * rounded(w, dtype)
    yd = dev(y, TORCH[dtype])
    update = ops.GatedNormedUpdate(ops.SummedRows(yd, pieces) if pieces > 1 else yd, dev(w_out, TORCH[dtype]), eps_out,
                                   dev(gate, TORCH[dtype])[:, :width] if gated else None, dev(bias) if gated else None)
    picked_stream = dev(x)
    picked = ops.gated_update_norm(update, picked_stream, dev(w, TORCH[dtype]), eps, rows=ints([5, 0, 5]))
    np.testing.assert_array_equal(picked_stream.cpu().numpy(), x)  # a row list leaves the stream as it is
    np.testing.assert_allclose(picked.float().cpu().numpy(), normed[[5, 0, 5]], rtol=0, atol=tolerance(dtype, 4))
    stream = dev(x)
    h = ops.gated_update_norm(update, stream, dev(w, TORCH[dtype]), eps)
    np.testing.assert_allclose(stream.cpu().numpy(), after, rtol=0, atol=5e-6)
    np.testing.assert_allclose(h.float().cpu().numpy(), normed, rtol=0, atol=tolerance(dtype, 4))
    np.testing.assert_allclose(update.finish().cpu().numpy(), after - x, rtol=0, atol=5e-6)  # for a norm that does not know it
    alone = ops.gated_update_norm(None, dev(x), dev(w, TORCH[dtype]), eps).float().cpu().numpy()
    want = x / np.sqrt((x.astype(np.float64) ** 2).mean(axis=1, keepdims=True) + eps) * rounded(w, dtype)
    np.testing.assert_allclose(alone, want, rtol=0, atol=tolerance(dtype, 4))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [10, 64, 1100, 5001])
@pytest.mark.parametrize("taps", [1, 2, 4, 6])
def test_single_tokens_pass_norm_and_convolution_in_one_launch(dtype, width, taps):
    """Five steps of single tokens of three requests in scattered slots (rows strided as in the engine's state
    buffer) and a padding row: the same rows as the norm and the convolution in turn, the same tails, and
    the plain convolution of each request's rows."""
    from mini_infer_amd import ops

    rng = np.random.default_rng(width + taps)
    slots, steps, seats = [2, -1, 4, 0], 5, 6
    taps_weight = rng.standard_normal((width, taps)).astype(np.float32)
    w = rng.uniform(0.5, 1.5, width).astype(np.float32)

    def tails():
        if taps == 1:
            return None
        wide = torch.zeros((seats + 1, (taps - 1) * width + 8), dtype=TORCH[dtype], device=DEV)
        return wide[:, : (taps - 1) * width].unflatten(1, (taps - 1, width))

    one, two = tails(), tails()
    seen = []
    for _ in range(steps):
        x = rng.standard_normal((4, width)).astype(np.float32)
        args = (dev(taps_weight), dev(taps_weight.T), one, ints(range(5)), ints(slots), ints(range(4)), True)
        h, u = ops.gated_update_norm(None, dev(x), dev(w, TORCH[dtype]), 1e-5, conv=ops.InputConvolution(*args))
        h2, u2 = ops.gated_update_norm(None, dev(x), dev(w, TORCH[dtype]), 1e-5,
                                       conv=ops.InputConvolution(*args[:2], two, *args[3:6], False))
        assert torch.equal(h, h2)
        np.testing.assert_allclose(u.float().cpu().numpy(), u2.float().cpu().numpy(), rtol=0, atol=tolerance(dtype, 2))
        seen.append((h.double().cpu().numpy(), u.double().cpu().numpy()))
        if taps > 1:
            assert torch.equal(one, two)
            assert not one[[1, 3, 5]].any()  # nobody else's rows
    for row in (0, 2, 3):
        h = np.stack([s[0][row] for s in seen])
        np.testing.assert_allclose(np.stack([s[1][row] for s in seen]), h + pf.causal_conv(h, taps_weight.astype(np.float64)), rtol=0,
                                   atol=tolerance(dtype, 8))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("channels, extra", [(8, 4), (10, 3), (64, 0), (1028, 4)])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5])
@pytest.mark.parametrize("add_input", [True, False])
def test_short_convolution_in_portions(dtype, channels, extra, taps, add_input):
    """Four requests over four steps: portions of one and two rows, shorter than the taps, longer than the
    walking kernel's limit and than a run of rows, request borders inside runs; a request that brings nothing."""
    from mini_infer_amd import ops

    rng = np.random.default_rng(channels + taps)
    weight = rng.standard_normal((channels, taps)).astype(np.float32)
    bias = rng.standard_normal(channels).astype(np.float32)
    lengths = {3: 140, 0: 29, 5: 61, 1: 8}  # by slot
    rows = {s: rng.standard_normal((n, channels + extra)).astype(np.float32) for s, n in lengths.items()}
    tail = torch.zeros((7, taps - 1, channels), dtype=TORCH[dtype], device=DEV)
    got = {s: [] for s in lengths}
    fed = {s: 0 for s in lengths}
    for step in ([(3, 2), (0, 1), (5, 3)], [(0, 17), (3, 100), (1, 2)], [(5, 58), (1, 0), (3, 1), (0, 9)], [(3, 37), (1, 6), (0, 2)]):
        x, cu, req = [], [0], []
        for b, (s, n) in enumerate(step):
            x.append(rows[s][fed[s]: fed[s] + n])
            cu.append(cu[-1] + n), req.extend([b] * n)
        y = ops.short_conv(dev(np.concatenate(x), TORCH[dtype]), channels, dev(weight), tail, ints(cu), ints([s for s, _ in step]), ints(req),
                           bias=dev(bias), add_input=add_input).double().cpu().numpy()
        for b, (s, n) in enumerate(step):
            got[s].append(y[cu[b]: cu[b + 1]])
            fed[s] += n
    assert fed == lengths
    for s in lengths:
        h = rounded(rows[s], dtype)[:, :channels]
        z = pf.causal_conv(h, weight.astype(np.float64)) + bias
        np.testing.assert_allclose(np.concatenate(got[s]), h + z if add_input else z / (1 + np.exp(-z)), rtol=0, atol=tolerance(dtype, 6))
    if taps > 1:
        for s in lengths:
            np.testing.assert_array_equal(tail[s].double().cpu().numpy(), rounded(rows[s], dtype)[-(taps - 1):, :channels])
        assert not tail[[2, 4, 6]].any()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tokens", [1, 16, 17, 70, 300])
@pytest.mark.parametrize("heads, k, n", [(3, 32, 16), (2, 96, 40), (5, 8, 7), (1, 130, 66), (4, 512, 128), (2, 24, 200)])
def test_a_product_head_by_head_with_and_without_a_gate(dtype, tokens, heads, k, n):
    from mini_infer_amd import ops

    rng = np.random.default_rng(tokens + k)
    head_width = k + 8
    x = rng.standard_normal((tokens, heads * head_width)).astype(np.float32)
    w = (rng.standard_normal((heads, n, k)) / np.sqrt(k)).astype(np.float32)
    gate = rng.standard_normal((tokens, heads * n + 8)).astype(np.float32) * 2
    xr, wr, gr = rounded(x, dtype).reshape(tokens, heads, head_width)[:, :, :k], rounded(w, dtype), rounded(gate, dtype)[:, : heads * n]
    want = np.einsum("thk,hnk->thn", xr, wr)
    view = dev(x, TORCH[dtype]).unflatten(1, (heads, head_width))[:, :, :k]
    wd = dev(w, TORCH[dtype])
    kn = wd.transpose(1, 2).contiguous() if tokens % 2 else None
    out = torch.zeros((tokens, heads, n + 2), dtype=TORCH[dtype], device=DEV)
    ops.linear_per_head(view, wd, out[:, :, :n], weight_kn=kn)
    np.testing.assert_allclose(out[:, :, :n].double().cpu().numpy(), want, rtol=0, atol=tolerance(dtype, 4))
    assert not out[:, :, n:].any()
    packed = torch.empty((tokens, heads * n), dtype=TORCH[dtype], device=DEV).unflatten(1, (heads, n))
    ops.linear_per_head(view, wd, packed, weight_kn=kn, gate=dev(gate, TORCH[dtype])[:, : heads * n].unflatten(1, (heads, n)))
    np.testing.assert_allclose(packed.double().cpu().numpy(), want / (1 + np.exp(-gr.reshape(tokens, heads, n))), rtol=0, atol=tolerance(dtype, 4))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads, padded, width", [(3, 24, 10), (1, 8, 8), (8, 192, 128)])
def test_heads_are_packed_and_gated(dtype, heads, padded, width):
    from mini_infer_amd import ops

    rng = np.random.default_rng(width)
    x = rng.standard_normal((9, heads * padded)).astype(np.float32)
    gate = rng.standard_normal((9, heads * width + 5)).astype(np.float32) * 3
    out = torch.empty((9, heads, width), dtype=TORCH[dtype], device=DEV)
    ops.gate_heads(dev(x, TORCH[dtype]).unflatten(1, (heads, padded)), dev(gate, TORCH[dtype])[:, : heads * width].unflatten(1, (heads, width)), out)
    want = rounded(x, dtype).reshape(9, heads, padded)[:, :, :width] / (1 + np.exp(-rounded(gate, dtype)[:, : heads * width].reshape(9, heads, width)))
    np.testing.assert_allclose(out.double().cpu().numpy(), want, rtol=0, atol=tolerance(dtype, 2))


def latent_reference(q, keys, positions, rank, scale, window, sinks):
    """[queries, heads, rank] for queries at `positions` over the keys up to each, NumPy float64."""
    out = np.zeros((q.shape[0], q.shape[1], rank))
    for i, p in enumerate(positions):
        lo = 0 if window is None else max(0, p - window + 1)
        s = keys[lo: p + 1] @ q[i].T * scale  # [keys, heads]
        top = np.maximum(s.max(axis=0), -np.inf if sinks is None else sinks)
        e = np.exp(s - top)
        total = e.sum(axis=0) + (0 if sinks is None else np.exp(sinks - top))
        out[i] = (e / total).T @ keys[lo: p + 1, :rank]
    return out


@pytest.mark.parametrize("heads, rank, rot, page, window, with_sinks", [
    (1, 16, 0, 4, None, False), (4, 80, 16, 16, None, False), (5, 48, 8, 8, 20, True), (17, 256, 32, 16, None, False),
    (20, 304, 24, 16, 37, False), (32, 512, 64, 16, None, False), (40, 512, 64, 32, 64, True), (3, 128, 64, 16, 1, False)])
def test_latent_rows_on_the_matrix_cores(heads, rank, rot, page, window, with_sinks):
    """Three requests of 343, 70 and 1 tokens in scattered pages (what lies behind a window marked as given back):
    as decoded tokens, as portions of unequal length, and with the boundaries known to the device only; keys cut into
    ranges and not.  The last query's first head singles out one key: far away at a page's border, or the last one
    inside the window, or (head two) the first one outside it, which must not show."""
    from mini_infer_amd import ops

    rng = np.random.default_rng(heads + rank)
    width, lengths, scale = rank + rot, [343, 70, 1], (rank + rot) ** -0.5
    keys = [rng.standard_normal((n, width)).astype(np.float32) for n in lengths]
    queries = [rng.standard_normal((n, heads, width)).astype(np.float32) for n in lengths]
    edge = page * 3 if window is None else lengths[0] - window
    queries[0][-1, 0] = 6.0 * keys[0][edge] / np.linalg.norm(keys[0][edge]) / (scale * np.sqrt(width))
    keys[0][edge] *= 4.0
    if window is not None and heads > 1:
        queries[0][-1, 1] = 6.0 * keys[0][edge - 1] / np.linalg.norm(keys[0][edge - 1]) / (scale * np.sqrt(width))
        keys[0][edge - 1] *= 4.0
    sinks = (rng.standard_normal(heads) * 2).astype(np.float32) if with_sinks else None
    counts = [-(-n // page) for n in lengths]
    order = rng.permutation(sum(counts) + 3)
    pages = np.zeros((sum(counts) + 3, 1, page, width), dtype=np.float32)
    table, at = np.full((3, max(counts) + 2), -1), 0
    for b, n in enumerate(lengths):
        for j in range(counts[b]):
            table[b, j] = order[at + j]
            piece = keys[b][j * page: (j + 1) * page]
            pages[order[at + j], 0, : len(piece)] = piece
        at += counts[b]
    kd = dev(pages, torch.bfloat16)
    for portion in ([1, 1, 1], [5, 33, 1], [0, 70, 1], [90, 1, 0]):
        starts = [n - q for n, q in zip(lengths, portion)]
        shown = table.copy()
        if window is not None:
            for b in range(3):
                shown[b, : max(0, starts[b] - window + 1) // page] = -1  # pages the window has passed
        q = np.concatenate([queries[b][starts[b]:] for b in range(3)])
        positions = np.concatenate([np.arange(starts[b], lengths[b]) for b in range(3)])
        cu = np.concatenate([[0], np.cumsum(portion)])
        want = np.concatenate([
            latent_reference(rounded(queries[b], "bfloat16")[starts[b]:], rounded(keys[b], "bfloat16"), range(starts[b], lengths[b]), rank, scale,
                             window, None if sinks is None else sinks.astype(np.float64)) for b in range(3)])
        qd = dev(q.reshape(len(q), heads * width), torch.bfloat16)
        for host in (cu.tolist(), None):
            for splits in (None, 1, 3, 16):
                got = ops.latent_attention(
                    qd, kd, ints(shown), ints(np.repeat(np.arange(3), portion)), ints(positions), ints(cu), host, heads=heads, rank=rank,
                    rot=rot, scale=scale, window=window, max_seq_len=343, sinks=None if sinks is None else dev(sinks), splits=splits,
                ).double().cpu().numpy().reshape(len(q), heads, rank)
                np.testing.assert_allclose(got, want, rtol=0, atol=2e-2 * max(1.0, np.abs(want).max()),
                                           err_msg=f"portions {portion}, host {host is not None}, ranges {splits}")
    first = latent_reference(rounded(queries[0], "bfloat16")[-1:], rounded(keys[0], "bfloat16"), [342], rank, scale, window, None)
    without = keys[0].copy()
    without[edge] = 0
    moved = latent_reference(rounded(queries[0], "bfloat16")[-1:], rounded(without, "bfloat16"), [342], rank, scale, window, None)
    assert window == 1 or np.abs(first - moved)[0, 0].max() > 0.3  # (the key that stands out is what the answer is made of)


def plain_experts(x, up, down, router, correction, top):
    """Ungated experts on stacked weights, logistic scores on what an expert reads (float64)."""
    out, chosen, weights = np.zeros((x.shape[0], down.shape[1])), [], []
    for t in range(x.shape[0]):
        z = router @ x[t]
        s = 1 / (1 + np.exp(-z))
        picks = np.argsort(-(z if correction is None else s + correction), kind="stable")[:top]
        chosen.append(picks), weights.append(s[picks])
        for e in picks:
            out[t] += down[e] @ (np.maximum(up[e] @ (s[e] * x[t]), 0) ** 2)
    return out, np.array(chosen), np.array(weights)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows, width, ff, experts, top, corrected", [
    (1, 24, 10, 3, 1, False), (9, 64, 48, 6, 2, True), (40, 90, 26, 5, 4, False), (70, 256, 128, 16, 4, True), (5, 48, 16, 1, 1, False),
    (3, 2048, 72, 4, 2, False), (130, 136, 40, 3, 2, False), (300, 128, 64, 70, 2, False), (515, 192, 320, 2, 1, False)])
def test_logistic_scores_and_all_forms_of_ungated_experts(dtype, rows, width, ff, experts, top, corrected):
    """The router's choice and weights against NumPy, then every form of the expert sum: pair by pair, expert by
    expert, in direct tiles, in tiles staged through LDS (rows left apart as well), sorted by expert; weights on the
    input and on the output; an expert that nobody chose."""
    from mini_infer_amd import ops

    rng = np.random.default_rng(rows * 7 + width)
    x = rng.standard_normal((rows, width)).astype(np.float32)
    router = (rng.standard_normal((experts, width)) * 2.0 / np.sqrt(width)).astype(np.float32)
    correction = (rng.standard_normal(experts) * 0.2).astype(np.float32) if corrected else None
    if corrected:
        correction[1] = -5.0
    up = (rng.standard_normal((experts, ff, width)) / np.sqrt(width) * 1.5).astype(np.float32)
    down = (rng.standard_normal((experts, width, ff)) / np.sqrt(ff)).astype(np.float32)
    xr, upr, downr = rounded(x, dtype), rounded(up, dtype), rounded(down, dtype)
    want, picks, scores = plain_experts(xr, upr, downr, router.astype(np.float64), correction, top)
    xd, ud, dd = dev(x, TORCH[dtype]), dev(up, TORCH[dtype]), dev(down, TORCH[dtype])
    chosen, w, none = ops.route_top_k(xd, dev(router), None if correction is None else dev(correction), None, top=top, route_scale=1.0,
                                      scores="logistic")
    np.testing.assert_array_equal(chosen.cpu().numpy(), picks)
    np.testing.assert_allclose(w.cpu().numpy(), scores, rtol=0, atol=2e-6)
    assert none is None and (not corrected or not (picks == 1).any())
    how = {"activation": "squared_relu", "weight_on": "input"}
    forms = {"few": lambda **k: ops.experts_few_rows(xd, ud, dd, chosen, w, **k), "grouped": lambda **k: ops.experts_grouped(xd, ud, dd, chosen, w, **k)}
    if ops.experts_by_expert_take(xd, ud, "squared_relu"):
        tiles = ["rows", "direct"] + (["lds"] if ops.expert_tiles_take(xd, ff) else [])
        forms.update({t: (lambda t: lambda **k: ops.experts_by_expert(xd, ud, dd, chosen, w, tiles=t, **k))(t) for t in tiles})
        forms["default"] = lambda **k: ops.experts_by_expert(xd, ud, dd, chosen, w, **k)
        for t in tiles:
            apart = ops.experts_by_expert(xd, ud, dd, chosen, w, tiles=t, combine=False, **how)
            assert isinstance(apart, ops.SummedRows) and apart.rows.shape == (rows * top, width)
            np.testing.assert_allclose(apart.finish().double().cpu().numpy(), want, rtol=0, atol=tolerance(dtype, 8) * max(1.0, np.abs(want).max()))
    assert "lds" in forms or dtype == "float32" or width % 64 or ff % 64
    # weights on the output: the weight enters once, not squared
    on_output = np.zeros_like(want)
    for t in range(rows):
        for e, s in zip(picks[t], scores[t]):
            on_output[t] += s * (downr[e] @ (np.maximum(upr[e] @ xr[t], 0) ** 2))
    for name, form in forms.items():
        got = form(**how).double().cpu().numpy()
        np.testing.assert_allclose(got, want, rtol=0, atol=tolerance(dtype, 8) * max(1.0, np.abs(want).max()), err_msg=name)
        got = form(activation="squared_relu", weight_on="output").double().cpu().numpy()
        np.testing.assert_allclose(got, on_output, rtol=0, atol=tolerance(dtype, 8) * max(1.0, np.abs(on_output).max()), err_msg=name)


@pytest.mark.parametrize("rows, width, ff, experts, identity, top", [(70, 256, 128, 16, 1, 4), (200, 64, 192, 3, 2, 2), (333, 128, 64, 5, 0, 1)])
def test_silu_gated_experts_in_tiles_staged_through_lds(rows, width, ff, experts, identity, top):
    from mini_infer_amd import ops

    rng = np.random.default_rng(rows)
    x = dev(rng.standard_normal((rows, width)), torch.bfloat16)
    gate_up = dev(rng.standard_normal((experts, 2 * ff, width)) / np.sqrt(width), torch.bfloat16)
    down = dev(rng.standard_normal((experts, width, ff)) / np.sqrt(ff), torch.bfloat16)
    router = dev(rng.standard_normal((experts + identity, width)) * 2 / np.sqrt(width))
    chosen, w, _ = ops.route_top_k(x, router, None, None, top=top, route_scale=1.5)
    want = ops.experts_few_rows(x, gate_up, down, chosen, w).double()
    got = ops.experts_by_expert(x, gate_up, down, chosen, w, tiles="lds").double()
    assert (got - want).abs().max() < 2e-2 * max(1.0, want.abs().max())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("scores", ["logistic", "softmax"])
@pytest.mark.parametrize("tokens, width, outputs, experts, top, corrected, gated", [
    (1, 64, 5, 5, 2, False, True), (8, 4096, 16, 16, 2, False, False), (13, 1028, 70, 66, 3, True, True), (32, 256, 200, 200, 7, True, False),
    (33, 256, 12, 10, 12, False, True), (9, 90, 6, 4, 2, True, True)])
def test_router_and_list_of_pairs_in_one_call(dtype, scores, tokens, width, outputs, experts, top, corrected, gated):
    """The same choices and weights as without the list, and every pair of a real expert listed once, under its expert."""
    from mini_infer_amd import ops

    rng = np.random.default_rng(tokens + width)
    x = dev(rng.standard_normal((tokens, width)), TORCH[dtype])
    router = dev(rng.standard_normal((outputs, width)) * 2.0 / np.sqrt(width))
    correction = dev(rng.standard_normal(outputs) * 0.2) if corrected else None
    gate_row = dev(rng.standard_normal(width) / np.sqrt(width)) if gated else None
    args, how = (x, router, correction, gate_row), {"top": top, "route_scale": 1.7, "scores": scores}
    chosen, weights, gates = ops.route_top_k(*args, **how)
    again = ops.route_top_k(*args, **how, experts=experts)
    assert torch.equal(chosen, again[0])
    np.testing.assert_allclose(again[1].cpu().numpy(), weights.cpu().numpy(), rtol=0, atol=4e-6)
    z = x.double().cpu().numpy() @ router.double().cpu().numpy().T
    s = 1 / (1 + np.exp(-z)) if scores == "logistic" else np.exp(z - z.max(axis=1, keepdims=True)) / np.exp(z - z.max(axis=1, keepdims=True)).sum(axis=1, keepdims=True)
    picks = np.argsort(-(s + (0 if correction is None else correction.double().cpu().numpy())), axis=1, kind="stable")[:, :top]
    np.testing.assert_array_equal(chosen.cpu().numpy(), picks)
    np.testing.assert_allclose(weights.cpu().numpy(), 1.7 * np.take_along_axis(s, picks, axis=1), rtol=0, atol=4e-6)
    if gated:
        np.testing.assert_allclose(again[2].cpu().numpy(), gates.cpu().numpy(), rtol=0, atol=2e-6)
    listed, first = again[3].listed.cpu().numpy(), again[3].first.cpu().numpy()
    flat = picks.reshape(-1)
    assert first[0] == 0 and first[-1] == (flat < experts).sum()
    for e in range(experts):
        assert sorted(listed[first[e]: first[e + 1]].tolist()) == np.flatnonzero(flat == e).tolist()


def test_logistic_scores_that_float32_cannot_tell_apart_are_ranked_by_their_logits():
    from mini_infer_amd import ops

    x = torch.ones((2, 4), device=DEV)
    router = dev(np.array([[5.0] * 4, [7.0] * 4, [6.0] * 4, [-9.0] * 4]))  # logits 20, 28, 24, -36: three scores round to one
    chosen, w, _ = ops.route_top_k(x, router, None, None, top=3, route_scale=1.0, scores="logistic")
    assert chosen.tolist() == [[1, 2, 0]] * 2
    np.testing.assert_allclose(w.cpu().numpy(), np.ones((2, 3)), rtol=0, atol=1e-6)


# ---------------------------------------------------------------------------------------------
# each part alone in a one-layer model
# ---------------------------------------------------------------------------------------------

ALONE = {
    "latent": tf.latent(3, 10, 6, 14, 22, 0.6, 50.0),
    "latent_fast": tf.latent(4, 16, 16, 24, 48, 0.3, 1000.0),
    "experts": tf.latent(2, 8, 4, 8, 16, 0.5, 30.0, tf.moe(24, 5, 3)),
    "experts_fast": tf.latent(2, 8, 8, 8, 16, 0.5, 30.0, tf.moe(64, 3, 2)),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("part", sorted(ALONE))
@pytest.mark.parametrize("taps", [1, 4])
def test_each_part_alone_whole_and_token_by_token(tmp_path, dtype, part, taps):
    from mini_infer_amd.engine import StepEntry

    cfg = tf.config(90, 64 if "fast" in part else 48, [ALONE[part]], eps=1e-5, taps=taps, scale=1.7)
    weights = tf.make_weights(cfg, seed=len(part), steady_choice=dtype == "bfloat16")
    folder = tf.write_model_dir(tmp_path / "m", cfg, weights)
    tokens = tf.random_tokens(cfg, 45, seed=9)
    want = oracle(f"{part}-{dtype}-{taps}", cfg, weights, tokens)
    runner = runner_for(folder, dtype, 8, pages=12, seats=2)
    whole = runner.step([StepEntry("w", tokens, list(range(45)))]).cpu().numpy()
    # (one layer, 45 tokens: the yardstick's largest error is the largest of few draws, so it gets more room)
    assert_close(whole, want, dtype, f"{part} whole", bf16_max_factor=3.0)
    one_by_one = np.concatenate([runner.step([StepEntry("d", [t], [0])]).cpu().numpy() for t in tokens])
    assert_close(one_by_one, want, dtype, f"{part} token by token", bf16_max_factor=3.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("gated, taps", [(False, 3), (True, None), (False, None)])
def test_a_sandwich_block_without_gates_or_without_convolutions(dtype, gated, taps):
    """The block's two mechanisms are each their own switch: a one-layer model as a `ModelSpec` of its own, against
    the plain model with gates of one (a bias that saturates them) or convolutions of zero."""
    import dataclasses

    from mini_infer_amd.engine import ModelRunner, StepEntry
    from mini_infer_amd.models import DecoderModel, architecture_for
    from mini_infer_amd.weights.loader import load_state_dict

    cfg = tf.config(80, 64, [tf.latent(3, 10, 6, 14, 22, 0.6, 50.0, tf.moe(24, 3, 2))], eps=1e-5, taps=taps or 2, scale=1.2)
    weights = tf.make_weights(cfg, seed=8, steady_choice=dtype == "bfloat16")
    plain = dict(weights)
    if not gated:
        for q in "12":
            plain.update({f"l0.rg{q}": np.zeros((64, 64), np.float32), f"l0.rg{q}.b": np.full(64, 40.0, np.float32)})
    if taps is None:
        plain.update({f"l0.canon{q}": np.zeros((64, 2), np.float32) for q in "12"})
    arch = architecture_for(cfg)
    parsed = arch.parse_config(cfg)
    spec = arch.build_spec(parsed)
    layer = dataclasses.replace(spec.layers[0], block={**spec.layers[0].block, "gated": gated, "conv_taps": taps})
    model = DecoderModel(dataclasses.replace(spec, layers=[layer]), TORCH[dtype], DEV)
    assert all((".rg" in name) <= gated and (".canon" in name) <= (taps is not None) for name in model.param_specs())
    load_state_dict(model, {k: torch.from_numpy(v) for k, v in weights.items() if k in model.param_specs()})
    runner = ModelRunner(model, parsed, num_blocks=16, block_size=8, max_concurrent=2)
    tokens = tf.random_tokens(cfg, 40, seed=2)
    want = oracle(f"sandwich-{dtype}-{gated}-{taps}", cfg, plain, tokens)
    got = np.concatenate([runner.step([StepEntry("a", part, list(range(len(part))))]).cpu().numpy()
                          for part in (tokens[:21], tokens[21:23], *[[t] for t in tokens[23:]])])
    assert_close(got, want, dtype, "sandwich", bf16_max_factor=3.0)


# ---------------------------------------------------------------------------------------------
# whole models under every kind of schedule
# ---------------------------------------------------------------------------------------------

LENGTHS = {"A": (70, 41, 9, 33, 58, 1), "B": (45, 64, 17, 2, 39), "C": (150, 40, 77, 5), "D": (50, 21, 36, 3, 44), "E": (90, 35, 3, 61)}


def requests_of(name, cfg):
    return {f"{name}{i}": tf.random_tokens(cfg, n, seed=100 * len(name) + 7 * i + n) for i, n in enumerate(LENGTHS[name])}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(tf.CONFIGS))
@pytest.mark.parametrize("family", ["whole", "decode", "portions", "mixed"])
def test_logits_do_not_depend_on_the_schedule(folders, name, dtype, family):
    """Whole prompts; a prompt and then its last tokens one by one; portions down to two tokens; up to four live
    requests of unequal length in one batch, in a pool so small that pages and state slots are used
    again.  Each request is held against itself alone."""
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
        # (a request of one or two tokens makes the yardstick's largest error the largest of few draws)
        assert_close(got[rid], oracle(name, cfg, weights, tokens), dtype, f"{name} {family} {rid}", bf16_max_factor=3.0 if len(tokens) < 10 else 2.0)
    runner.cache.check()
    assert runner.cache.states.num_free == runner.cache.states.max_requests
    assert runner.num_free_blocks() == pages


@pytest.mark.parametrize("dtype", DTYPES)
def test_several_prompts_begin_in_one_step_and_go_on_in_portions_beside_single_tokens(folders, dtype):
    """C's sizes: a step in which every request begins writes keys and values out per head (bfloat16), a step
    of many rows takes the expert tiles, later portions run over the cache; recorded and not."""
    from mini_infer_amd.engine import StepEntry
    from mini_infer_amd.parts.latent_attention import LatentAttention

    name, cfg, block, weights, folder = folders["C", dtype]
    first, second, third = (tf.random_tokens(cfg, n, seed=n) for n in (190, 83, 61))
    calls = {"expanded": 0}
    original = LatentAttention._forward_expanded

    def counted(self, *args, **kwargs):
        calls["expanded"] += 1
        return original(self, *args, **kwargs)

    for graphs in (True, False):
        runner = runner_for(folder, dtype, block, pages=24, seats=3, graphs=graphs)
        LatentAttention._forward_expanded = counted
        calls["expanded"] = 0
        try:
            both = runner.step([StepEntry("a", first[:100], list(range(100))), StepEntry("b", second[:50], list(range(50)))]).cpu().numpy()
        finally:
            LatentAttention._forward_expanded = original
        assert calls["expanded"] == (4 if dtype == "bfloat16" else 0)
        got = {"a": [both[:100]], "b": [both[100:]], "c": []}
        steps = [{"a": (100, 101), "c": (0, 60), "b": (50, 52)}, {"a": (101, 190), "b": (52, 53)}, {"b": (53, 83), "c": (60, 61)}]
        for step in steps:
            entries = [StepEntry(r, {"a": first, "b": second, "c": third}[r][i:j], list(range(j - i))) for r, (i, j) in step.items()]
            logits = runner.step(entries).cpu().numpy()
            at = 0
            for r, (i, j) in step.items():
                got[r].append(logits[at: at + j - i])
                at += j - i
        for r, tokens in (("a", first), ("b", second), ("c", third)):
            assert_close(np.concatenate(got[r]), oracle(name, cfg, weights, tokens), dtype, f"{r}, recorded {graphs}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_slot_and_pages_used_again_start_clean(folders, dtype):
    """One seat, pages for one request: the second request gets the first one's slot (with the first one's
    last rows in its tails) and pages."""
    from mini_infer_amd.engine import StepEntry

    name, cfg, block, weights, folder = folders["A", dtype]
    first, second = tf.random_tokens(cfg, 30, seed=1), tf.random_tokens(cfg, 26, seed=2)
    runner = runner_for(folder, dtype, block, pages=2, seats=1)
    runner.step([StepEntry("a", first, [])])
    slot = runner.cache.state_slot("a")
    runner.free_request("a")
    got = runner.step([StepEntry("b", second[:2], [0, 1])]).cpu().numpy()
    assert runner.cache.state_slot("b") == slot
    got = np.concatenate([got, runner.step([StepEntry("b", second[2:], list(range(24)))]).cpu().numpy()])
    assert_close(got, oracle(name, cfg, weights, second), dtype, "second owner of a slot")


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_step_that_fails_leaves_the_tails_as_they_were(folders, dtype, monkeypatch):
    """A step whose last layer refuses after every convolution has moved its tails on: the same step goes through
    afterwards as if nothing had been tried."""
    from mini_infer_amd.engine import StepEntry

    name, cfg, block, weights, folder = folders["A", dtype]
    tokens = tf.random_tokens(cfg, 40, seed=3)
    runner = runner_for(folder, dtype, block, pages=4, seats=1, graphs=False)
    got = [runner.step([StepEntry("a", tokens[:11], list(range(11)))]).cpu().numpy()]
    head = runner.model.head

    def refuse(*args, **kwargs):
        raise RuntimeError("refused")

    for part in (tokens[11:13], tokens[13:14], tokens[14:40]):
        monkeypatch.setattr(head, "forward", refuse)
        with pytest.raises(RuntimeError, match="refused"):
            runner.step([StepEntry("a", part, [0])])
        monkeypatch.undo()
        got.append(runner.step([StepEntry("a", part, list(range(len(part))))]).cpu().numpy())
    assert_close(np.concatenate(got), oracle(name, cfg, weights, tokens), dtype, "after refused steps")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "E"])
def test_long_decoding_through_recorded_steps(folders, dtype, name):
    """Two requests decoded side by side for 150 steps after prompts of 130 and 7 tokens, across many page
    borders; the single-token steps are replayed graphs, with eager work between them."""
    from mini_infer_amd.engine import StepEntry

    name, cfg, block, weights, folder = folders[name, dtype]
    requests = {"x": tf.random_tokens(cfg, 280, seed=31), "y": tf.random_tokens(cfg, 157, seed=32)}
    runner = runner_for(folder, dtype, block, pages=34, seats=3)
    got = {rid: [] for rid in requests}
    both = runner.step([StepEntry("x", requests["x"][:130], list(range(130))), StepEntry("y", requests["y"][:7], list(range(7)))]).cpu().numpy()
    got["x"].append(both[:130])
    got["y"].append(both[130:])
    for k in range(150):
        if k in (20, 70):  # a prompt of another request between the replays
            runner.step([StepEntry("z", tf.random_tokens(cfg, 40, seed=k), [39])])
            runner.free_request("z")
        logits = runner.step([StepEntry("x", [requests["x"][130 + k]], [0]), StepEntry("y", [requests["y"][7 + k]], [0])]).cpu().numpy()
        got["x"].append(logits[:1])
        got["y"].append(logits[1:])
    assert runner.decode_graphs is not None and runner.decode_graphs.replays == 150
    for rid, tokens in requests.items():
        assert_close(np.concatenate(got[rid]), oracle(name, cfg, weights, tokens), dtype, f"long decoding {rid}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("fast", [True, False])
def test_one_far_key_is_found_by_prompts_portions_and_decoded_tokens(tmp_path, dtype, fast):
    """One layer whose first head singles out one token far back: at the sequence's start, at page borders and
    inside.  The plain model says that replacing that token moves the last logits by far more than
    any tolerance; the engine agrees with both sequences in a whole prompt, in portions and decoded."""
    from mini_infer_amd.engine import StepEntry

    layer = tf.latent(3, 16, 16, 16, 48, 0.3, 100.0) if fast else tf.latent(3, 10, 6, 14, 22, 0.3, 100.0)
    m = layer["mixer"]
    cfg = tf.config(60, 64, [layer], eps=1e-5, taps=2, scale=1.0)
    weights = tf.make_weights(cfg, seed=12)
    key_token, query_token, d = 58, 59, m["dim"] + m["rot_dim"]
    weights["embed"][:, 1:3] = 0.0
    weights["embed"][key_token, 1] = weights["embed"][query_token, 2] = 4.0
    weights["l0.norm1"][1:3] = 1.0
    weights["l0.canon1"][1:3] = 0.0
    weights["l0.mix.dkv"][0] = 0.0  # the latent's first entry reads the key token alone, and the first head's
    weights["l0.mix.dkv"][0, 1] = 4.0  # first key entry and query entry meet there
    weights["l0.mix.uk"][0] = 0.0
    weights["l0.mix.uk"][0, 0] = 4.0
    weights["l0.mix.q"][0] = 0.0
    weights["l0.mix.q"][0, 2] = 4.0
    assert weights["l0.mix.q"].shape[0] == 3 * d
    folder = tf.write_model_dir(tmp_path / "m", cfg, {k: tf.bf16_round(v) for k, v in weights.items()})
    weights = {k: tf.bf16_round(v) for k, v in weights.items()}
    base = [t % 58 for t in tf.random_tokens(cfg, 330, seed=4)]
    base[-1] = query_token
    runner = runner_for(folder, dtype, 16, pages=24, seats=1)
    plain = oracle(f"far-{fast}-none", cfg, weights, base)
    for place in (0, 1, 15, 16, 31, 32, 200, 271, 272, 328):
        tokens = list(base)
        tokens[place] = key_token
        want = oracle(f"far-{fast}-{place}", cfg, weights, tokens)
        shows = float(np.abs(want.exact[-1] - plain.exact[-1]).max())
        assert shows > 5 * max(plain.yard_p99, 0.01), f"key at {place}: {shows:.3f} against {plain.yard_p99:.3f}"
        runs = {"whole": [tokens], "portions": [tokens[:40], tokens[40:42], tokens[42:329], tokens[329:]], "decoded": [tokens[:325]] + [[t] for t in tokens[325:]]}
        for how, portions in runs.items():
            for part in portions:
                logits = runner.step([StepEntry(how, part, [len(part) - 1])]).cpu().numpy()
            runner.free_request(how)
            last = want[slice(329, 330)]
            last.moved_by_float32 = want.moved_by_float32
            assert_close(logits, last, dtype, f"{how}, key at {place}", bf16_max_factor=3.0)


@pytest.mark.parametrize("name", ["A", "B"])
def test_greedy_generation_through_llm_and_the_scheduler(folders, name):
    """Five prompts for two seats, prompts cut into portions of 8 under a 20-token budget: every generated token
    is the plain model's greedy choice."""
    from mini_infer_amd.engine.llm import LLM

    _, cfg, block, weights, folder = folders[name, "float32"]
    wide = {k: v.astype(np.float64) for k, v in weights.items()}
    lengths, new_tokens = (5, 19, 33, 2, 11), 9
    prompts = [tf.random_tokens(cfg, n, seed=300 + n) for n in lengths]
    llm = LLM(folder, dtype="float32", num_blocks=12, block_size=block, max_concurrent=2, max_num_batched_tokens=20, chunk_size=8)
    results = llm.generate(prompts, max_tokens=new_tokens)
    for prompt, result in zip(prompts, results):
        sequence = list(prompt)
        for _ in range(new_tokens):
            sequence.append(pf.greedy(pf.logits(cfg, wide, sequence)[-1]))
        assert result.tokens == sequence[len(prompt):] and result.finish_reason == "length"
    assert llm.runner.cache.states.num_free == 2
    llm.runner.cache.check()


def test_the_command_line_writes_random_weights_and_generates_greedily_and_by_seeded_sampling(tmp_path, capsys):
    """`random-weights` from a config.json, then `generate`: greedy twice the same, sampled with one seed twice
    the same and (at this temperature) different from greedy."""
    from mini_infer_amd.__main__ import main

    cfg, block = tf.CONFIGS["A"]
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
    requests = {f"t{i}": tf.random_tokens(cfg, n, seed=i) for i, n in enumerate((70, 41, 9, 33, 58))}
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
