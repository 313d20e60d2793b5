"""Figosun configurations drawn by seed: sizes, head counts, taps, shared tensors, experts, constants, layer
order and page size all vary; each is run whole and under a mixed schedule (four live requests, pools
used again) and held against the plain model, in both engines (bfloat16 with steadily chosen experts: see
`tiny_figosun.make_weights`)."""

import numpy as np
import pytest

import plain_figosun as pf
import replay_util as ru
import tiny_figosun as tf

pytestmark = pytest.mark.gpu
SEEDS = list(range(14))
CHAOTIC_SHARE = 0.02  # of the largest |logit|: a yardstick whose 99th percentile lies beyond this says nothing


def draw(seed: int):
    rng = np.random.default_rng(3000 + seed)
    pick = lambda values: values[int(rng.integers(0, len(values)))]  # noqa: E731
    width = pick([40, 48, 64, 72, 90, 96, 128, 192, 200, 256])

    def mlp():
        if rng.random() < 0.25:
            return None
        experts = pick([1, 2, 3, 5, 8, 16])
        return tf.moe(pick([16, 26, 32, 64, 72, 128]), experts, int(rng.integers(1, min(experts, 5) + 1)))

    layers = []
    for n in range(int(rng.integers(1, 6))):
        if n and rng.random() < 0.35:
            layers.append(tf.again(layers, int(rng.integers(0, n))))
            continue
        heads, dim, rot = pick([1, 2, 3, 4, 6, 8, 20]), pick([4, 8, 16, 24, 32, 48, 64]), pick([2, 4, 8, 16, 32, 64])
        layers.append(tf.latent(heads, dim, rot, pick([4, 8, 16, 24, 32, 64, 80]), pick([8, 12, 32, 48, 64, 96, 128, 144, 256]),
                                float(rng.uniform(0.5, 1.5)) * (dim + rot) ** -0.5, float(pick([10.0, 1000.0, 20000.0, 1e6])), mlp()))
    cfg = tf.config(int(rng.integers(60, 400)), width, layers, eps=float(pick([1e-6, 1e-5, 1e-4])), taps=int(rng.integers(1, 7)),
                    scale=float(pick([0.5, 1.0, 3.0, 8.0])))
    return cfg, pick([4, 8, 16, 16, 32])


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def get(seed, dtype):
        if (seed, dtype) not in made:
            cfg, block = draw(seed)
            weights = tf.make_weights(cfg, seed=seed, steady_choice=dtype == "bfloat16")
            folder = tf.write_model_dir(tmp_path_factory.mktemp("random") / f"{seed}-{dtype}", cfg, weights)
            lengths = (101, 3, 38, 1, 55)
            requests = {f"q{i}": tf.random_tokens(cfg, n, seed=seed * 10 + i) for i, n in enumerate(lengths)}
            wide = {k: v.astype(np.float64) for k, v in weights.items()}
            oracles = {}
            for rid, t in requests.items():
                exact = pf.logits(cfg, wide, t)
                oracles[rid] = ru.Oracle(exact, pf.logits(cfg, wide, t, store=pf.bf16_round))
                pf.ANGLE_TYPE = np.float32  # (a float32 engine's angles: see plain_figosun)
                try:
                    as_float32 = pf.logits(cfg, wide, t, store=pf.f32_round)
                finally:
                    pf.ANGLE_TYPE = np.float64
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
