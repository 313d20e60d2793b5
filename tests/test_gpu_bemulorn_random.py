"""Bemulorn configurations drawn by seed: sizes, head counts, chunks, rotations, shared keys, experts, constants,
layer order and page size all vary; each is run whole and under a mixed schedule (four live requests, pools
used again) and held against the plain model, in both engines (bfloat16 with steadily chosen experts: see
`tiny_bemulorn.make_weights`)."""

import numpy as np
import pytest

import plain_bemulorn as pb
import replay_util as ru
import tiny_bemulorn as tb

pytestmark = pytest.mark.gpu
SEEDS = list(range(16))
CHAOTIC_SHARE = 0.02  # of the largest |logit|: a yardstick whose 99th percentile lies beyond this says nothing


def draw(seed: int):
    rng = np.random.default_rng(5000 + seed)
    pick = lambda values: values[int(rng.integers(0, len(values)))]  # noqa: E731
    width = pick([40, 48, 64, 72, 90, 96, 128, 192, 224, 320])

    def mlp():
        kind = rng.random()
        if kind < 0.15:
            return None
        if kind < 0.55:
            return tb.dense(pick([24, 40, 64, 70, 96, 160, 192]), float(rng.uniform(0.6, 5.0)))
        experts = pick([1, 2, 3, 5, 8, 16])
        return tb.moe(pick([16, 26, 32, 64, 72, 128]), experts, int(rng.integers(1, min(experts, 5) + 1)), pick([None, 16, 30, 64, 96]))

    layers = []
    for n in range(int(rng.integers(1, 6))):
        own = [i for i, layer in enumerate(layers) if "kv_from" not in layer["mixer"]]
        chunk = pick([None, 1, 3, 8, 16, 29, 32, 64, 90, 200])
        if own and rng.random() < 0.4:
            source = pick(own)
            m = layers[source]["mixer"]
            layers.append(tb.attention(m["kv_heads"] * pick([1, 2, 3, 4]), m["kv_heads"], m["dim"], m["vdim"], m["scale"] * pick([0.8, 1.0, 1.3]),
                                       m.get("mask", {}).get("size") if rng.random() < 0.5 else chunk, m.get("rot"), mlp(), source))
            continue
        kv_heads, dim = pick([1, 2, 3]), pick([4, 8, 18, 24, 32, 64, 96, 128])
        rot = None
        if rng.random() < 0.85:
            dims = 2 * int(rng.integers(1, dim // 2 + 1)) if rng.random() < 0.5 else dim
            scaling = None if rng.random() < 0.3 else (float(rng.uniform(1.0, 16.0)), int(rng.integers(16, 400)), float(rng.uniform(2.0, 40.0)), float(rng.uniform(0.3, 2.0)))
            rot = tb.rotation(float(pick([10.0, 1000.0, 20000.0, 1e6])), dims, scaling)
        layers.append(tb.attention(kv_heads * pick([1, 2, 3, 5, 8]), kv_heads, dim, pick([4, 8, 14, 16, 32, 48, 64, 80, 128]),
                                   float(rng.uniform(0.4, 1.0)) * dim ** -0.5, chunk, rot, mlp()))
    cfg = tb.config(int(rng.integers(60, 400)), width, layers, eps=float(pick([1e-6, 1e-5, 1e-4])), scale=float(pick([0.5, 1.0, 3.0, 8.0])),
                    logit_scale=float(pick([0.25, 1.0, 2.5])), positions=int(rng.integers(101, 400)))
    return cfg, pick([4, 8, 16, 16, 16, 32])


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def get(seed, dtype):
        if (seed, dtype) not in made:
            cfg, block = draw(seed)
            weights = tb.make_weights(cfg, seed=seed, steady_choice=dtype == "bfloat16")
            folder = tb.write_model_dir(tmp_path_factory.mktemp("random") / f"{seed}-{dtype}", cfg, weights)
            lengths = (101, 3, 38, 1, 55)
            requests = {f"q{i}": tb.random_tokens(cfg, n, seed=seed * 10 + i) for i, n in enumerate(lengths)}
            wide = {k: v.astype(np.float64) for k, v in weights.items()}
            oracles = {}
            for rid, t in requests.items():
                exact = pb.logits(cfg, wide, t)
                oracles[rid] = ru.Oracle(exact, pb.logits(cfg, wide, t, store=pb.bf16_round))
                pb.ANGLE_TYPE = np.float32  # (a float32 engine's angles: see plain_bemulorn)
                try:
                    as_float32 = pb.logits(cfg, wide, t, store=pb.f32_round)
                finally:
                    pb.ANGLE_TYPE = np.float64
                oracles[rid].moved_by_float32 = float(np.abs(as_float32 - exact).max())
            made[seed, dtype] = (cfg, block, folder, requests, oracles)
        return made[seed, dtype]

    return get


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("family", ["whole", "mixed"])
@pytest.mark.parametrize("seed", SEEDS)
def test_a_configuration_drawn_by_seed(models, seed, family, dtype):
    from mini_infer_amd.engine import ModelRunner

    cfg, block, folder, requests, oracles = models(seed, dtype)
    schedule = ru.schedule_whole(requests) if family == "whole" else ru.schedule_mixed(requests, seed=seed, max_live=4, tail=9)
    pages = ru.peak_pages(requests, schedule, block)
    runner = ModelRunner.from_pretrained(folder, dtype=dtype, num_blocks=pages, block_size=block, max_concurrent=4)
    got = ru.run_schedule(runner, requests, schedule)
    what = f"seed {seed} ({len(cfg['layers'])} layers, width {cfg['width']}, pages of {block})"
    for rid in requests:
        if dtype == "bfloat16" and oracles[rid].yard_p99 > CHAOTIC_SHARE * float(np.abs(oracles[rid].exact).max()):
            continue  # (bfloat16 storage alone scatters this configuration's logits: nothing to hold an engine against)
        # float32: 1e-4, or twice as far as float32 storage and angles alone move this input's logits; bfloat16: three
        # times the yardstick's largest error (requests of 1 and 3 tokens make it the largest of few draws)
        ru.assert_close(got[rid], oracles[rid], dtype, f"{what} {family} {rid}",
                        fp32_tol=max(ru.FP32_TOL, 2.0 * oracles[rid].moved_by_float32), bf16_max_factor=3.0)
    runner.cache.check()
    assert runner.cache.states.num_free == 4 and runner.num_free_blocks() == pages
