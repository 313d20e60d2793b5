"""Bemulorn without a GPU: configuration, the model as data (tensor names, shared keys and values, cache
needs, joint products), the pages chunks give back, the frequency table, and the plain model against itself
(every mechanism matters; a prompt's prefix does not see what follows; chunks end where they should)."""

import copy
import json
import math

import numpy as np
import pytest
import torch

import plain_bemulorn as pb
import tiny_bemulorn as tb
from mini_infer_amd.cache.manager import RELEASED, CacheManager
from mini_infer_amd.exceptions import ConfigError
from mini_infer_amd.models import architecture_for
from mini_infer_amd.parts.base import CacheNeeds, PagedKVNeeds


def model_of(cfg, dtype=torch.bfloat16):
    arch = architecture_for(cfg)
    return arch.make_model(arch.parse_config(cfg), dtype, "cpu")


@pytest.mark.parametrize("name", sorted(tb.CONFIGS))
def test_the_model_asks_for_exactly_the_checkpoints_tensors(name):
    cfg, _ = tb.CONFIGS[name]
    specs = model_of(cfg).param_specs()
    assert {k: tuple(v.shape) for k, v in specs.items()} == tb.tensor_shapes(cfg)
    # what is added to a float32 sum and what makes a router's logits stays 32-bit whatever the engine's dtype
    assert all(v.dtype == "float32" for k, v in specs.items() if k.endswith((".b", "mlp.router")))


def test_layers_without_keys_of_their_own_read_their_source_and_ask_for_nothing():
    cfg, block = tb.CONFIGS["A"]
    model = model_of(cfg)
    assert [call.reads_cache_of for call in model.spec.order] == [None, 0, None, 0, 2]
    needs = model.cache_needs(block)
    assert [need is None for need in needs] == [False, True, False, True, True]
    first, third = needs[0].pages, needs[2].pages
    assert (first.num_kv_heads, first.head_dim, first.value_dim) == (2, 16, 24)
    # a reader with another chunk: nothing of the first layer's pages can be given back; the third's readers agree
    assert first.chunk is None and third.chunk == 50 and first.window is None
    assert not first.v_transposed  # (heads of 16: the plain kernel)


def test_value_heads_of_their_own_width_lie_transposed_where_the_matrix_core_kernel_reads_them():
    needs = model_of(tb.CONFIGS["C"][0]).cache_needs(16)
    assert needs[0].pages.v_transposed and (needs[0].pages.head_dim, needs[0].pages.value_dim) == (64, 112)
    assert needs[1].pages.v_transposed and (needs[1].pages.head_dim, needs[1].pages.value_dim) == (96, 48)
    assert not model_of(tb.CONFIGS["C"][0]).cache_needs(32)[0].pages.v_transposed  # (pages of 16 slots only)
    assert not model_of(tb.CONFIGS["C"][0], torch.float32).cache_needs(16)[0].pages.v_transposed


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0].update(type="recurrent"), "type"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "multiple"),
    (lambda c: c["layers"][0]["mixer"].pop("dim"), "dim"),
    (lambda c: c["layers"][0]["mixer"].update(scale=0), "scale"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5), "dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("fast"), "fast"),
    (lambda c: c["layers"][1]["mixer"].update(kv_from=1), "earlier"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=1), "keys and values of its own"),
    (lambda c: c["layers"][4]["mixer"].update(kv_from=0), "other key/value heads"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(base=301.0), "rotation"),
    (lambda c: c["layers"][1]["mlp"].update(kind="sparse"), "mlp"),
    (lambda c: c["layers"][1]["mlp"].pop("limit"), "limit"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=7), "top"),
    (lambda c: c["norm"].update(eps=0), "eps"),
    (lambda c: c.pop("embedding"), "embedding"),
    (lambda c: c.update(max_positions=0), "max_positions"),
])
def test_configurations_the_design_does_not_have_are_refused(change, message):
    cfg = json.loads(json.dumps(tb.CONFIGS["A"][0]))  # (layers of the tiny configuration share objects)
    change(cfg)
    with pytest.raises(ConfigError, match=message):
        architecture_for(cfg).parse_config(cfg)


def test_a_reader_may_leave_out_what_equals_its_source():
    cfg = json.loads(json.dumps(tb.CONFIGS["A"][0]))
    for key in ("kv_heads", "dim", "vdim", "rot"):
        del cfg["layers"][1]["mixer"][key]
    parse = architecture_for(cfg).parse_config
    assert parse(cfg) == parse(tb.CONFIGS["A"][0])


def test_the_number_of_positions_may_be_the_tables_alone():
    cfg = {k: v for k, v in tb.CONFIGS["D"][0].items() if k != "max_positions"}
    arch = architecture_for(cfg)
    parsed = arch.with_checkpoint_shapes(arch.parse_config(cfg), {"pos": (77, 48)})
    assert arch.make_model(parsed, torch.float32, "cpu").num_positions == 77
    with pytest.raises(ConfigError, match="max_positions"):
        arch.build_spec(arch.parse_config(cfg))


def test_joint_products_are_stacked_once_and_the_parts_keep_views_of_them():
    cfg, _ = tb.CONFIGS["A"]
    weights = {k: torch.from_numpy(v) for k, v in tb.make_weights(cfg, seed=3).items()}
    model = model_of(cfg, torch.float32)
    model.load_params(lambda name: weights[name])
    routed, dense, bare = model.blocks[0], model.blocks[1], model.blocks[2]
    # [q 64 | k 32 | v 48 | gates 4 and 4 rows of zeros | the shared expert's gate and up]; [o 96 | down 40]
    assert routed.joint.partner is routed.feed_forward.shared and routed.beside is routed.feed_forward
    stacked = routed.joint.input_weight
    assert stacked.shape == (64 + 32 + 48 + 8 + 80, 64) and routed.joint.output_weight.shape == (64, 96 + 40)
    assert torch.equal(stacked[144:148], weights["l0.mix.g"]) and not stacked[148:152].any()
    assert torch.equal(routed.feed_forward.shared.gate_up.weight, torch.cat([weights["l0.mlp.shared.gate"], weights["l0.mlp.shared.up"]]))
    assert routed.feed_forward.shared.gate_up.weight.data_ptr() == stacked[152:].data_ptr()
    assert torch.equal(routed.mixer.out.weight, weights["l0.mix.o"]) and torch.equal(routed.feed_forward.shared.down.weight, weights["l0.mlp.shared.down"])
    # a reader's rows: its queries, gates and the feed-forward alone
    assert dense.joint.layout.kv_heads == 0 and dense.joint.input_weight.shape[0] == 96 + 8 + 160 and dense.beside is None
    assert torch.equal(dense.mixer.bias, weights["l1.mix.q.b"])
    assert torch.equal(bare.mixer.bias, torch.cat([weights[f"l2.mix.{n}.b"] for n in "qkv"]))
    assert bare.joint.partner is None and bare.beside is None
    # dense layers hand their last product on, routed ones (whose norm's output the router reads) do not
    assert dense.emit_pending_output and dense.norm.emit_scaled_rows and not routed.norm.emit_scaled_rows
    # configurations of other designs whose blocks are parallel are built as before
    assert all(getattr(b, "joint", None) is not None for b in model.blocks)


def test_pages_of_chunks_that_have_ended_are_given_back():
    needs = [CacheNeeds(pages=PagedKVNeeds(1, 4, chunk=10))]
    cache = CacheManager(needs, page_size=4, num_pages=6, max_requests=2, allocate_storage=False)
    cache.add_request("a")
    held = []
    for _ in range(33):
        cache.reserve({"a": 1})
        index = cache.build_step_index([("a", 1)])
        length, table = int(index.seq_lens[0]), index.block_tables[0][0]
        # every key of the token's own chunk is there
        first = (length - 1) // 10 * 10
        assert all(table[p // 4] != RELEASED for p in range(first, length))
        cache.commit({"a": 1})
        cache.check()
        held.append(6 - cache.num_free_pages())
        # what the next token cannot see is not held
        assert all(p == RELEASED for p in cache.groups[0].tables["a"][: length // 10 * 10 // 4])
    assert max(held) <= 4 and held[19] <= 1 and held[29] == 1  # (a chunk that has ended holds at most the page its successor begins in)
    cache.free_request("a")
    assert cache.num_free_pages() == 6
    # calls with other chunks are another group
    both = CacheManager([needs[0], CacheNeeds(pages=PagedKVNeeds(1, 4, chunk=12)), CacheNeeds(pages=PagedKVNeeds(1, 4))],
                        page_size=4, num_pages=6, max_requests=2, allocate_storage=False)
    assert [group.chunk for group in both.groups] == [10, 12, None] and [group.releases for group in both.groups] == [True, True, False]


@pytest.mark.parametrize("rot", [tb.YARN_A, tb.YARN_C, tb.rotation(50.0, 24, (2.5, 32, 3.0, 0.5)), tb.rotation(1000.0, 6, (9.0, 20, 30.0, 2.0)),
                                 tb.rotation(20.0, 4), tb.rotation(7.0, 2, (1.0, 100, 5.0, 5.0)), tb.rotation(100.0, 64, (16.0, 4096, 1e6, 1e-3))])
def test_the_engines_frequencies_are_the_plain_ones(rot):
    from mini_infer_amd.parts.position import RotaryPosition

    part = RotaryPosition(rot["dims"], rot["base"], torch.float32, "cpu", exact_frequencies=True, yarn=rot.get("scaling"))
    turns, amplitude = pb.frequencies(rot)
    np.testing.assert_allclose(part.inv_freq_host.numpy(), np.array(turns), rtol=1e-7)
    assert math.isclose(part.amplitude, amplitude, rel_tol=1e-12)
    if rot.get("scaling") is None or rot["scaling"]["factor"] == 1.0:
        assert part.amplitude == 1.0


def test_a_blend_keeps_fast_pairs_divides_slow_ones_and_is_linear_between():
    turns, _ = pb.frequencies(tb.YARN_C)
    plain, _ = pb.frequencies({k: v for k, v in tb.YARN_C.items() if k != "scaling"})
    ratio = np.array(turns) / np.array(plain)
    inside = ratio[(ratio < 1) & (ratio > 0.125 + 1e-9)]
    assert ratio[0] == 1.0 and math.isclose(ratio[-1], 0.125) and len(inside) >= 2
    np.testing.assert_allclose(np.diff(inside), np.diff(inside)[0], rtol=1e-9)


def logits_of(cfg, weights, tokens):
    return pb.logits(cfg, {k: v.astype(np.float64) for k, v in weights.items()}, tokens)


def test_every_mechanism_of_the_tiny_weights_matters():
    """A constant or a tensor left out moves the plain model's logits by far more than any tolerance."""
    cfg, _ = tb.CONFIGS["A"]
    weights = tb.make_weights(cfg, seed=70)
    tokens = tb.random_tokens(cfg, 60, seed=4)
    base = logits_of(cfg, weights, tokens)

    def moved(other_cfg=None, **tensors):
        return np.abs(logits_of(other_cfg or cfg, {**weights, **tensors}, tokens) - base).max()

    for name in ("l0.norm1", "l2.norm1", "final.norm"):
        assert moved(**{name: np.ones_like(weights[name])}) > 0.05, name
    for name in ("pos", "l0.mix.q.b", "l0.mix.k.b", "l0.mix.v.b", "l1.mix.q.b", "l0.mix.g", "l1.mix.g", "l4.mix.g", "l0.mlp.router.b",
                 "l0.mlp.shared.down", "l3.mlp.router.b", "l1.mlp.up"):
        assert moved(**{name: np.zeros_like(weights[name])}) > 0.05, name
    assert moved({**cfg, "embedding": {"scale": 2.0}}) > 0.05 and moved({**cfg, "logit_scale": 1.7}) > 0.05
    for layer, key, value in ((0, "scale", 0.55), (4, "scale", 0.33), (1, "mask", {"size": 32}), (2, "mask", {"size": 49}),
                              (0, "rot", {"base": 300.0, "dims": 12}), (2, "rot", tb.rotation(50.0, 24, (2.5, 32, 3.0, 0.7))),
                              (2, "rot", tb.rotation(50.0, 24, (2.5, 32, 2.0, 0.5)))):
        other = copy.deepcopy(cfg)
        other["layers"][layer]["mixer"][key] = value
        assert moved(other) > 1e-2, (layer, key)
    for layer, key, value in ((1, "limit", 1.7), (4, "limit", 100.0)):
        other = copy.deepcopy(cfg)
        other["layers"][layer]["mlp"][key] = value
        assert moved(other) > 1e-3, (layer, key)
    other = copy.deepcopy(cfg)
    other["layers"][0]["mlp"]["router"]["top"] = 1
    assert moved(other) > 0.05


def test_a_reader_uses_its_sources_keys_and_values_with_a_mask_of_its_own():
    """What layer 0 makes of its keys moves layer 1 (chunk 33 over layer 0's keys, whose own chunk is 20): a
    key that layer 0 itself no longer sees."""
    cfg, _ = tb.CONFIGS["A"]
    cfg = {**cfg, "layers": cfg["layers"][:2]}
    weights = {k: v for k, v in tb.make_weights(tb.CONFIGS["A"][0], seed=9).items() if not k.startswith(("l2", "l3", "l4"))}
    tokens = tb.random_tokens(cfg, 33, seed=1)
    other = list(tokens)
    other[3] = (tokens[3] + 1) % cfg["vocab"]  # in layer 0's first chunk, 0 .. 19; positions 20 .. 32 see it in layer 1 only
    moved = np.abs(logits_of(cfg, weights, tokens) - logits_of(cfg, weights, other))
    assert moved[20:].max() > 0.01
    alone = copy.deepcopy(cfg)
    alone["layers"][1]["mixer"]["mask"]["size"] = 20
    moved = np.abs(logits_of(alone, weights, tokens) - logits_of(alone, weights, other))
    assert moved[:20].max() > 0.01 and moved[20:].max() == 0.0


def test_one_is_added_to_the_denominator():
    scores = np.array([-1.0, 0.5, 2.0])
    np.testing.assert_allclose(pb.softmax_plus_one(scores), np.exp(scores) / (1 + np.exp(scores).sum()), rtol=1e-14)
    np.testing.assert_allclose(pb.softmax_plus_one(np.array([800.0, 799.0])).sum(), 1.0, rtol=1e-12)
    assert pb.softmax_plus_one(np.array([-50.0])).sum() < 1e-20


def test_a_prefix_does_not_see_what_follows():
    cfg, _ = tb.CONFIGS["C"]
    weights = tb.make_weights(cfg, seed=5)
    tokens = tb.random_tokens(cfg, 30, seed=6)
    np.testing.assert_allclose(logits_of(cfg, weights, tokens[:11]), logits_of(cfg, weights, tokens)[:11], rtol=0, atol=1e-10)


def test_steadily_chosen_experts_are_far_from_a_close_call():
    for name in ("A", "B", "C", "D"):
        cfg, _ = tb.CONFIGS[name]
        pb.CHOICE_MARGINS = []
        try:
            logits_of(cfg, tb.make_weights(cfg, seed=70, steady_choice=True), tb.random_tokens(cfg, 60, seed=1))
            assert min(pb.CHOICE_MARGINS) > 0.8, (name, min(pb.CHOICE_MARGINS))
        finally:
            pb.CHOICE_MARGINS = None


def test_parts_refuse_what_they_do_not_build():
    from mini_infer_amd.parts.attention import GQAttention
    from mini_infer_amd.parts.joint import JointProducts

    with pytest.raises(NotImplementedError, match="head norms"):
        GQAttention(64, 4, 2, 16, None, torch.bfloat16, "cpu", head_norm={"eps": 1e-5}, bias_suffix=".b")
    with pytest.raises(NotImplementedError, match="one number per head"):
        GQAttention(64, 4, 2, 16, None, torch.bfloat16, "cpu", gate={"name": "g", "activation": "silu", "per_head": True})
    wide_gate = GQAttention(64, 4, 2, 16, None, torch.bfloat16, "cpu", gate={"name": "g"})
    with pytest.raises(ValueError, match="made together"):
        JointProducts(wide_gate, None, torch.bfloat16)
