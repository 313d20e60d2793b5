"""Figosun without a GPU: configuration, the model as data (tensor names, shared tensors, cache needs),
and the plain model against itself (every mechanism matters; a prompt's prefix does not see what follows)."""

import copy

import numpy as np
import pytest
import torch

import plain_figosun as pf
import tiny_figosun as tf
from mini_infer_amd.exceptions import ConfigError
from mini_infer_amd.models import architecture_for


def model_of(cfg, dtype=torch.bfloat16):
    arch = architecture_for(cfg)
    return arch.make_model(arch.parse_config(cfg), dtype, "cpu")


@pytest.mark.parametrize("name", sorted(tf.CONFIGS))
def test_the_model_asks_for_exactly_the_checkpoints_tensors(name):
    cfg, _ = tf.CONFIGS[name]
    specs = model_of(cfg).param_specs()
    assert {k: tuple(v.shape) for k, v in specs.items()} == tf.tensor_shapes(cfg)
    # what enters a router, a convolution's sum or a gate's sum beside the product stays 32-bit whatever the engine's dtype
    for leaf in ("canon1", "canon2", "rg1.b", "rg2.b", "mix.dkv.norm", "mlp.router"):
        assert all(v.dtype == "float32" for k, v in specs.items() if k.endswith(leaf))


def test_layers_that_share_tensors_are_one_block_with_a_cache_and_state_each():
    cfg, block = tf.CONFIGS["B"]  # layers 2 and 3 run with layer 1's tensors (3 through 2), layer 4 with layer 0's
    model = model_of(cfg)
    assert [call.layer for call in model.spec.order] == [0, 1, 1, 1, 0] and len(model.blocks) == 2
    assert all(call.reads_cache_of is None for call in model.spec.order)
    needs = model.cache_needs(block)
    assert len(needs) == 5
    for need, layer in zip(needs, cfg["layers"]):
        m = layer["mixer"]  # one row [latent | rotated part] per token, no value pages, no window
        assert (need.pages.num_kv_heads, need.pages.head_dim, need.pages.value_dim, need.pages.window) == (1, m["kv_rank"] + m["rot_dim"], 0, None)
        assert {name: state.shape for name, state in need.state.items()} == {"mixer_conv": (1, 90), "ffn_conv": (1, 90)}
        assert all(state.dtype == torch.bfloat16 for state in need.state.values())


def test_a_layer_without_feed_forward_keeps_one_tail_and_one_tap_needs_none():
    needs = model_of(tf.CONFIGS["A"][0]).cache_needs(16)
    assert sorted(needs[0].state) == ["ffn_conv", "mixer_conv"] and sorted(needs[1].state) == ["mixer_conv"]
    assert needs[1].state["mixer_conv"].shape == (3, 64)
    assert all(need.state is None and need.pages is not None for need in model_of(tf.CONFIGS["D"][0]).cache_needs(4))


def test_a_checkpoint_may_store_the_second_sublayers_tensors_of_a_layer_that_has_none():
    model = model_of(tf.CONFIGS["A"][0])
    assert {"l1.norm2", "l1.norm2b", "l1.canon2", "l1.rg2", "l1.rg2.b"} <= model.optional_names()
    assert "l0.norm2" not in model.optional_names()


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0].update(type="attention"), "type"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=4), "rot_dim"),
    (lambda c: c["layers"][1]["mixer"].pop("kv_rank"), "kv_rank"),
    (lambda c: c["layers"][3]["mixer"].update(scale=0), "scale"),
    (lambda c: c["layers"][3]["mlp"].update(kind="dense"), "mlp"),
    (lambda c: c["layers"][3]["mlp"]["router"].update(top=9), "top"),
    (lambda c: c["layers"][2].update(weights_of=7), "weights_of"),
    (lambda c: c["layers"][2].update(weights_of=2), "itself"),
    (lambda c: (c["layers"][0].update(weights_of=2)), "itself"),
    (lambda c: c["layers"][2].update(weights_of=1), "other sizes"),
    (lambda c: c["canon"].update(taps=0), "taps"),
    (lambda c: c["norm"].update(eps=0), "eps"),
    (lambda c: c.pop("embedding"), "embedding"),
])
def test_configurations_the_design_does_not_have_are_refused(change, message):
    cfg = copy.deepcopy(tf.CONFIGS["A"][0])
    change(cfg)
    with pytest.raises(ConfigError, match=message):
        architecture_for(cfg).parse_config(cfg)


def test_parts_refuse_what_they_do_not_build():
    from mini_infer_amd.parts.feed_forward import RoutedExperts

    with pytest.raises(NotImplementedError, match="weights on"):
        RoutedExperts(64, 32, 4, 2, torch.bfloat16, "cpu", weight_on="input")  # silu-gated experts
    with pytest.raises(NotImplementedError, match="scores"):
        RoutedExperts(64, 32, 4, 2, torch.bfloat16, "cpu", scores="max")
    with pytest.raises(NotImplementedError, match="identity"):
        RoutedExperts(64, 32, 4, 2, torch.bfloat16, "cpu", activation="squared_relu", weight_on="input", identity=1)


def logits_of(cfg, weights, tokens):
    return pf.logits(cfg, {k: v.astype(np.float64) for k, v in weights.items()}, tokens)


def test_every_mechanism_of_the_tiny_weights_matters():
    """A constant or a tensor left out moves the plain model's logits by far more than any tolerance."""
    cfg, _ = tf.CONFIGS["A"]
    weights = tf.make_weights(cfg, seed=70)
    tokens = tf.random_tokens(cfg, 60, seed=4)
    base = logits_of(cfg, weights, tokens)

    def moved(other_cfg=None, **tensors):
        return np.abs(logits_of(other_cfg or cfg, {**weights, **tensors}, tokens) - base).max()

    for name in ("l0.norm1", "l0.norm2", "l0.norm1b", "l0.norm2b", "l1.norm1b", "final.norm", "l0.mix.dkv.norm", "l3.mix.dkv.norm"):
        assert moved(**{name: np.ones_like(weights[name])}) > 0.05, name
    for name in ("l0.canon1", "l0.canon2", "l1.canon1", "l3.canon2", "l0.rg1", "l0.rg2", "l0.rg1.b", "l3.rg2.b", "l0.mix.g", "l1.mix.g"):
        assert moved(**{name: np.zeros_like(weights[name])}) > 0.05, name
    assert moved(**{"l0.canon1": weights["l0.canon1"][:, ::-1].copy()}) > 0.05  # the taps' order
    assert moved({**cfg, "embedding": {"scale": 2.5}}) > 0.05
    for layer, key, value in ((0, "scale", 0.45), (3, "scale", 0.45), (1, "rot", {"base": 900.0, "dims": 8})):
        other = copy.deepcopy(cfg)
        other["layers"][layer]["mixer"][key] = value
        assert moved(other) > 1e-2, (layer, key)
    other = copy.deepcopy(cfg)
    other["layers"][0]["mlp"]["router"]["top"] = 1
    assert moved(other) > 0.05
    other = copy.deepcopy(cfg)
    other["layers"][2] = {**other["layers"][1], "weights_of": 1}  # the third layer with other tensors
    assert moved(other) > 0.05


def test_the_weight_multiplies_what_an_expert_reads():
    rng = np.random.default_rng(0)
    width, ff = 12, 6
    w = {"router": rng.standard_normal((2, width))}
    for e in range(2):
        w.update({f"e{e}.up": rng.standard_normal((ff, width)), f"e{e}.down": rng.standard_normal((width, ff))})
    h = rng.standard_normal((4, width))
    got = pf.routed_feed_forward(h, w, tf.moe(ff, 2, 2))
    want = np.zeros_like(h)
    for e in range(2):
        s = 1 / (1 + np.exp(-(h @ w["router"][e])))
        want += (s ** 2)[:, None] * (np.maximum(h @ w[f"e{e}.up"].T, 0) ** 2 @ w[f"e{e}.down"].T)  # the square is of degree two
    np.testing.assert_allclose(got, want, rtol=0, atol=1e-12)


def test_a_prefix_does_not_see_what_follows_and_the_first_tokens_read_zeros():
    cfg, _ = tf.CONFIGS["C"]
    weights = tf.make_weights(cfg, seed=5)
    tokens = tf.random_tokens(cfg, 30, seed=6)
    np.testing.assert_allclose(logits_of(cfg, weights, tokens[:11]), logits_of(cfg, weights, tokens)[:11], rtol=0, atol=1e-10)
    h = np.arange(8, dtype=np.float64).reshape(4, 2) + 1
    taps = np.array([[1.0, 10.0, 100.0], [2.0, 20.0, 200.0]])
    np.testing.assert_array_equal(pf.causal_conv(h, taps), [[100, 400], [310, 840], [531, 1284], [753, 1728]])


def test_steadily_chosen_experts_are_far_from_a_close_call():
    for name in ("A", "B", "C", "E"):
        cfg, _ = tf.CONFIGS[name]
        pf.CHOICE_MARGINS = []
        try:
            logits_of(cfg, tf.make_weights(cfg, seed=70, steady_choice=True), tf.random_tokens(cfg, 60, seed=1))
            assert min(pf.CHOICE_MARGINS) > 0.2, (name, min(pf.CHOICE_MARGINS))
        finally:
            pf.CHOICE_MARGINS = None
