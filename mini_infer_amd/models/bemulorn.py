"""Bemulorn as a `ModelSpec`: a stack whose layers are listed in config.json one by one.  A layer is
parallel: one RMS norm, and both the mixer and the feed-forward (where the layer has one) read its output
and are added to the stream together, so their products are made together too (`joint`).  The
mixer is grouped-query attention inside chunks of positions: biases on queries, keys and values, a
partial rotation (halves paired) with frequencies rescaled the YaRN way, a softmax with one added to
its denominator, and one gate per head on what it attended to.  A layer may have no keys and values
of its own and read those of an earlier layer, with its own queries, chunk and everything else.  Two
feed-forwards: a dense clamped gated one and a mixture of experts (biased logits, weights by the softmax
over the chosen logits, a shared expert).  In front a scaled embedding plus a learned row per
position, behind a norm and a head whose logits are scaled.

config.json gives every size and every constant that differs between models of the design (`vocab`,
`width`, `max_positions`, `embedding.scale`, `logit_scale`, `norm.eps`, and per layer `type`, `mixer`
and `mlp`); tensor names are the checkpoint's own (`embed`, `pos`, `l<i>.{norm1,mix.*,mlp.*}`,
`final.norm`, `head`).  A key that config.json does not hold switches its mechanism off.
"""

from __future__ import annotations

import dataclasses
from typing import Any

from mini_infer_amd.exceptions import ConfigError
from mini_infer_amd.models.spec import Architecture, LayerCall, LayerSpec, ModelSpec
from mini_infer_amd.registry import ARCHITECTURES

NAME = "Bemulorn"
MIXER_TYPES = ("attention",)
FEED_FORWARD_KINDS = ("dense", "moe")
SINK_LOGIT = 0.0  # the softmax's denominator holds exp(0) beside the keys' terms
POSITION_TABLE = "pos"


def _positive_int(where: str, value: Any) -> int:
    if isinstance(value, bool) or not isinstance(value, int) or value <= 0:
        raise ConfigError(f"{where} must be a positive integer, got {value!r}")
    return value


def _number(where: str, value: Any) -> float:
    if isinstance(value, bool) or not isinstance(value, (int, float)):
        raise ConfigError(f"{where} must be a number, got {value!r}")
    return float(value)


def _positive(where: str, value: Any) -> float:
    number = _number(where, value)
    if not number > 0:
        raise ConfigError(f"{where} must be positive, got {number}")
    return number


def _section(raw: dict[str, Any], key: str, where: str = "config.json") -> dict[str, Any]:
    value = raw.get(key)
    if not isinstance(value, dict):
        raise ConfigError(f"{where} needs an object under {key!r}")
    return value


@dataclasses.dataclass(frozen=True)
class Stretch:
    """How a rotation's frequencies are rescaled."""

    factor: float
    original: float
    fast: float
    slow: float


@dataclasses.dataclass(frozen=True)
class Rotation:
    base: float
    dims: int
    scaling: Stretch | None = None


@dataclasses.dataclass(frozen=True)
class Experts:
    ff: int
    experts: int
    top: int
    shared_ff: int | None = None


@dataclasses.dataclass(frozen=True)
class BemulornLayer:
    type: str
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int | None = None
    rot: Rotation | None = None
    kv_from: int | None = None  # the layer whose keys and values this one reads
    dense_ff: int | None = None  # a dense feed-forward, with its limit
    limit: float | None = None
    moe: Experts | None = None  # a mixture of experts (neither: the layer has no feed-forward)


@dataclasses.dataclass(frozen=True)
class BemulornConfig:
    architecture: str
    vocab: int
    width: int
    max_positions: int | None  # None: as many as the checkpoint's table of positions has rows
    embedding_scale: float
    logit_scale: float
    norm_eps: float
    layers: tuple[BemulornLayer, ...]

    @classmethod
    def from_dict(cls, raw: dict[str, Any]) -> "BemulornConfig":
        entries = raw.get("layers")
        if not isinstance(entries, list) or not entries:
            raise ConfigError("config.json needs a non-empty list under 'layers'")
        layers = tuple(_parse_layer(f"layers[{i}]", _with_sources_sizes(entry, entries)) for i, entry in enumerate(entries))
        for i, layer in enumerate(layers):
            _check_source(i, layer, layers)
        return cls(
            architecture=str(raw.get("architecture") or (raw.get("architectures") or [NAME])[0]),
            vocab=_positive_int("vocab", raw.get("vocab")),
            width=_positive_int("width", raw.get("width")),
            max_positions=None if raw.get("max_positions") is None else _positive_int("max_positions", raw["max_positions"]),
            embedding_scale=_number("embedding.scale", _section(raw, "embedding").get("scale")),
            logit_scale=_number("logit_scale", raw.get("logit_scale", 1.0)),
            norm_eps=_positive("norm.eps", _section(raw, "norm").get("eps")),
            layers=layers,
        )


def _with_sources_sizes(entry: Any, entries: list) -> Any:
    """A layer that reads another's keys and values may leave out what has to equal that layer's."""
    mixer = entry.get("mixer") if isinstance(entry, dict) else None
    source = mixer.get("kv_from") if isinstance(mixer, dict) else None
    if not isinstance(source, int) or isinstance(source, bool) or not 0 <= source < len(entries) or not isinstance(entries[source], dict):
        return entry
    theirs = entries[source].get("mixer")
    if not isinstance(theirs, dict):
        return entry
    return {**entry, "mixer": {**{key: theirs[key] for key in ("kv_heads", "dim", "vdim", "rot") if key in theirs}, **mixer}}


def _check_source(i: int, layer: BemulornLayer, layers: tuple[BemulornLayer, ...]) -> None:
    """A layer that reads another's keys and values: that one comes earlier, has its own, and fits."""
    if layer.kv_from is None:
        return
    where = f"layers[{i}].mixer.kv_from"
    if not 0 <= layer.kv_from < i:
        raise ConfigError(f"{where} must name an earlier layer, got {layer.kv_from}")
    source = layers[layer.kv_from]
    if source.kv_from is not None:
        raise ConfigError(f"{where} names layer {layer.kv_from}, which has no keys and values of its own")
    mine, theirs = [(x.kv_heads, x.dim, x.vdim, x.rot) for x in (layer, source)]
    if mine != theirs:
        raise ConfigError(f"{where}: layer {layer.kv_from} has other key/value heads, widths or another rotation: {theirs}, not {mine}")


def _parse_rotation(at: str, mixer: dict[str, Any], dim: int) -> Rotation | None:
    if mixer.get("rot") is None:
        return None
    rot = _section(mixer, "rot", at)
    dims = _positive_int(f"{at}.rot.dims", rot.get("dims"))
    if dims % 2 or dims > dim:
        raise ConfigError(f"{at}.rot.dims={dims} must be even and at most {dim}")
    base = _positive(f"{at}.rot.base", rot.get("base"))
    scaling = None
    if rot.get("scaling") is not None:
        section = _section(rot, "scaling", f"{at}.rot")
        scaling = Stretch(*(_positive(f"{at}.rot.scaling.{key}", section.get(key)) for key in ("factor", "original", "fast", "slow")))
        if base == 1.0:
            raise ConfigError(f"{at}.rot.base must not be 1 where frequencies are rescaled")
    return Rotation(base, dims, scaling)


def _parse_layer(where: str, entry: Any) -> BemulornLayer:
    if not isinstance(entry, dict):
        raise ConfigError(f"{where} must be an object")
    kind = entry.get("type")
    if kind not in MIXER_TYPES:
        raise ConfigError(f"{where}.type is {kind!r}; this design has {MIXER_TYPES}")
    mixer = _section(entry, "mixer", where)
    at = f"{where}.mixer"
    fields: dict[str, Any] = {"type": kind}
    for key in ("heads", "dim"):
        fields[key] = _positive_int(f"{at}.{key}", mixer.get(key))
    fields["kv_heads"] = _positive_int(f"{at}.kv_heads", mixer.get("kv_heads", fields["heads"]))
    fields["vdim"] = _positive_int(f"{at}.vdim", mixer.get("vdim", fields["dim"]))
    if fields["heads"] % fields["kv_heads"] != 0:
        raise ConfigError(f"{where}: heads={fields['heads']} is not a multiple of kv_heads={fields['kv_heads']}")
    fields["scale"] = _positive(f"{at}.scale", mixer.get("scale"))
    if mixer.get("mask") is not None:
        fields["chunk"] = _positive_int(f"{at}.mask.size", _section(mixer, "mask", at).get("size"))
    fields["rot"] = _parse_rotation(at, mixer, fields["dim"])
    source = mixer.get("kv_from")
    if source is not None:
        if isinstance(source, bool) or not isinstance(source, int):
            raise ConfigError(f"{at}.kv_from must be a layer's number, got {source!r}")
        fields["kv_from"] = source
    mlp = entry.get("mlp")
    if mlp is not None:
        if not isinstance(mlp, dict) or mlp.get("kind") not in FEED_FORWARD_KINDS:
            raise ConfigError(f"{where}.mlp must be null or an object of kind {FEED_FORWARD_KINDS}, got {mlp!r}")
        if mlp["kind"] == "dense":
            fields["dense_ff"] = _positive_int(f"{where}.mlp.ff", mlp.get("ff"))
            fields["limit"] = _positive(f"{where}.mlp.limit", mlp.get("limit"))
        else:
            router = _section(mlp, "router", f"{where}.mlp")
            fields["moe"] = Experts(
                ff=_positive_int(f"{where}.mlp.expert.ff", _section(mlp, "expert", f"{where}.mlp").get("ff")),
                experts=_positive_int(f"{where}.mlp.router.experts", router.get("experts")),
                top=_positive_int(f"{where}.mlp.router.top", router.get("top")),
                shared_ff=None if mlp.get("shared") is None
                else _positive_int(f"{where}.mlp.shared.ff", _section(mlp, "shared", f"{where}.mlp").get("ff")),
            )
            if fields["moe"].top > fields["moe"].experts:
                raise ConfigError(f"{where}.mlp.router: top={fields['moe'].top} of {fields['moe'].experts} experts")
    return BemulornLayer(**fields)


def with_checkpoint_shapes(cfg: BemulornConfig, shapes: dict) -> BemulornConfig:
    """Where config.json does not say how many positions there are, the checkpoint's table of them does."""
    if cfg.max_positions is None and POSITION_TABLE in shapes:
        return dataclasses.replace(cfg, max_positions=int(shapes[POSITION_TABLE][0]))
    return cfg


def _cache_chunk(cfg: BemulornConfig, i: int) -> int | None:
    """The chunk behind which layer i's pages can be given back: its own, where every layer that reads
    its keys and values has the same one."""
    readers = [layer.chunk for layer in cfg.layers if layer.kv_from == i]
    return cfg.layers[i].chunk if all(chunk == cfg.layers[i].chunk for chunk in readers) else None


def bemulorn_spec(cfg: BemulornConfig) -> ModelSpec:
    if cfg.max_positions is None:
        raise ConfigError("max_positions is neither in config.json nor known from a checkpoint's table of positions")
    norm = {"kind": "rms_norm", "hidden_size": cfg.width, "eps": cfg.norm_eps, "name": ""}
    names = {"norm": "norm1", "mixer": "mix.", "feed_forward": "mlp."}
    layers, order = [], []
    for i, layer in enumerate(cfg.layers):
        mixer: dict[str, Any] = {
            "kind": "gqa_attention", "hidden_size": cfg.width, "num_heads": layer.heads, "num_kv_heads": layer.kv_heads,
            "head_dim": layer.dim, "v_head_dim": layer.vdim, "scale": layer.scale, "sink_logit": SINK_LOGIT, "chunk": layer.chunk,
            "names": ("q", "k", "v", "o"), "suffix": "", "bias_suffix": ".b", "own_keys": layer.kv_from is None,
            "cache_chunk": _cache_chunk(cfg, i),
            "gate": {"name": "g", "activation": "logistic", "per_head": True},
            "position": None,
        }
        if layer.rot is not None:
            # exact_frequencies: powers and rescaling evaluated in 64-bit before they become the float32 table
            mixer["position"] = {"kind": "rotary", "head_dim": layer.dim, "theta": layer.rot.base, "rotary_dim": layer.rot.dims,
                                 "interleaved": False, "exact_frequencies": True}
            if layer.rot.scaling is not None:
                mixer["position"]["yarn"] = dataclasses.asdict(layer.rot.scaling)
        feed_forward = None
        if layer.dense_ff is not None:
            feed_forward = {"kind": "clamped_glu", "hidden_size": cfg.width, "intermediate_size": layer.dense_ff,
                            "limit": layer.limit, "biases": False}
        elif layer.moe is not None:
            feed_forward = {"kind": "routed_experts", "hidden_size": cfg.width, "intermediate_size": layer.moe.ff,
                            "experts": layer.moe.experts, "top": layer.moe.top, "scores": "chosen_softmax", "correction": True,
                            "names": {"correction": "router.b"}, "shared_size": layer.moe.shared_ff, "shared_gated": False}
        block = {"kind": "parallel", "norm": norm, "mixer": mixer, "feed_forward": feed_forward, "joint": True, "names": names}
        layers.append(LayerSpec(prefix=f"l{i}.", block=block))
        order.append(LayerCall(i, reads_cache_of=layer.kv_from))
    return ModelSpec(
        vocab_size=cfg.vocab,
        hidden_size=cfg.width,
        layers=layers,
        order=order,
        final_norm={**norm, "name": "norm"},
        final_norm_prefix="final.",
        max_position_embeddings=cfg.max_positions,
        embedding={"kind": "learned_position_embedding", "vocab_size": cfg.vocab, "hidden_size": cfg.width, "name": "embed",
                   "scale": cfg.embedding_scale, "position_name": POSITION_TABLE, "num_positions": cfg.max_positions},
        head={"kind": "linear_head", "vocab_size": cfg.vocab, "hidden_size": cfg.width, "name": "head", "tied": False,
              "scale": cfg.logit_scale},
    )


BEMULORN = ARCHITECTURES.register(NAME, Architecture(
    name=NAME, parse_config=BemulornConfig.from_dict, build_spec=bemulorn_spec, with_checkpoint_shapes=with_checkpoint_shapes))
