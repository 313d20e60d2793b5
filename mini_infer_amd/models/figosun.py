"""Figosun as a `ModelSpec`: a stack whose layers are listed in config.json one by one.  A layer is a
mixer and, where it has one, a feed-forward, each between two RMS norms: `x <- x + norm_b(gate *
sublayer(u))`, where `h = norm(x)`, `u = h + conv(h)` with a short causal convolution per channel, and
`gate = logistic(W h + b)` element by element.  The mixer is attention over a low-rank latent (rotated
key part shared by the heads, no window) whose heads' outputs are gated by the mixer's input; the
feed-forward is a mixture of ungated squared-relu experts with logistic scores that multiply what an
expert reads.  A layer may run with another layer's tensors (`weights_of`), with a cache and state of
its own.  In front a scaled embedding; behind a norm and the embedding table as head.

config.json gives every size and every constant that differs between models of the design (`vocab`,
`width`, `norm.eps`, `canon.taps`, `embedding.scale`, and per layer `type`, `mixer`, `mlp` and
`weights_of`); tensor names are the checkpoint's own (`embed`, `l<i>.{norm1,norm1b,canon1,rg1,rg1.b,
mix.*,norm2,norm2b,canon2,rg2,rg2.b,mlp.*}`, `final.norm`).
"""

from __future__ import annotations

import dataclasses
from typing import Any

from mini_infer_amd.exceptions import ConfigError
from mini_infer_amd.models.spec import Architecture, LayerCall, LayerSpec, ModelSpec
from mini_infer_amd.registry import ARCHITECTURES

NAME = "Figosun"
MIXER_TYPES = ("latent_attention",)
FEED_FORWARD_KINDS = ("moe",)


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
    if number <= 0:
        raise ConfigError(f"{where} must be positive, got {number}")
    return number


def _section(raw: dict[str, Any], key: str, where: str = "config.json") -> dict[str, Any]:
    value = raw.get(key)
    if not isinstance(value, dict):
        raise ConfigError(f"{where} needs an object under {key!r}")
    return value


@dataclasses.dataclass(frozen=True)
class Experts:
    ff: int
    experts: int
    top: int


@dataclasses.dataclass(frozen=True)
class FigosunLayer:
    type: str
    heads: int
    dim: int  # unrotated part of a query or key head
    rot_dim: int  # rotated part, all of it rotated
    rot_base: float
    vdim: int
    kv_rank: int
    scale: float
    moe: Experts | None = None  # None: the layer has no feed-forward


@dataclasses.dataclass(frozen=True)
class FigosunConfig:
    architecture: str
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    taps: int
    layers: tuple[FigosunLayer, ...]
    # for every layer the one whose tensors it runs with (itself, unless the file says otherwise)
    owners: tuple[int, ...]

    @classmethod
    def from_dict(cls, raw: dict[str, Any]) -> "FigosunConfig":
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json needs a non-empty list under 'layers'")
        parsed = tuple(_parse_layer(f"layers[{i}]", entry) for i, entry in enumerate(layers))
        owners = tuple(_owner(layers, i) for i in range(len(layers)))
        for i, owner in enumerate(owners):
            if parsed[i] != parsed[owner]:
                raise ConfigError(f"layers[{i}] runs with the tensors of layers[{owner}] but describes other sizes")
        return cls(
            architecture=str(raw.get("architecture") or (raw.get("architectures") or [NAME])[0]),
            vocab=_positive_int("vocab", raw.get("vocab")),
            width=_positive_int("width", raw.get("width")),
            norm_eps=_positive("norm.eps", _section(raw, "norm").get("eps")),
            embedding_scale=_number("embedding.scale", _section(raw, "embedding").get("scale")),
            taps=_positive_int("canon.taps", _section(raw, "canon").get("taps")),
            layers=parsed,
            owners=owners,
        )


def _owner(layers: list, index: int) -> int:
    """The layer whose tensors layer `index` runs with: `weights_of` followed to its end."""
    seen = [index]
    while layers[seen[-1]].get("weights_of") is not None:
        target = layers[seen[-1]]["weights_of"]
        if isinstance(target, bool) or not isinstance(target, int) or not 0 <= target < len(layers):
            raise ConfigError(f"layers[{seen[-1]}].weights_of must name one of the {len(layers)} layers, got {target!r}")
        if target in seen:
            raise ConfigError(f"layers[{index}].weights_of leads back to itself: {seen + [target]}")
        seen.append(target)
    return seen[-1]


def _parse_layer(where: str, entry: Any) -> FigosunLayer:
    if not isinstance(entry, dict):
        raise ConfigError(f"{where} must be an object")
    kind = entry.get("type")
    if kind not in MIXER_TYPES:
        raise ConfigError(f"{where}.type is {kind!r}; this design has {MIXER_TYPES}")
    mixer, at = _section(entry, "mixer", where), f"{where}.mixer"
    fields: dict[str, Any] = {"type": kind}
    for key in ("heads", "dim", "rot_dim", "vdim", "kv_rank"):
        fields[key] = _positive_int(f"{at}.{key}", mixer.get(key))
    fields["scale"] = _positive(f"{at}.scale", mixer.get("scale"))
    rot = _section(mixer, "rot", at)
    fields["rot_base"] = _positive(f"{at}.rot.base", rot.get("base"))
    dims = _positive_int(f"{at}.rot.dims", rot.get("dims"))
    if dims != fields["rot_dim"] or dims % 2:
        raise ConfigError(f"{at}: the rotated part is rot_dim={fields['rot_dim']} wide (even) and all of it is rotated, got rot={rot!r}")
    mlp = entry.get("mlp")
    if mlp is not None:
        if not isinstance(mlp, dict) or mlp.get("kind") not in FEED_FORWARD_KINDS:
            raise ConfigError(f"{where}.mlp must be null or an object of kind {FEED_FORWARD_KINDS}, got {mlp!r}")
        router = _section(mlp, "router", f"{where}.mlp")
        moe = Experts(
            ff=_positive_int(f"{where}.mlp.expert.ff", _section(mlp, "expert", f"{where}.mlp").get("ff")),
            experts=_positive_int(f"{where}.mlp.router.experts", router.get("experts")),
            top=_positive_int(f"{where}.mlp.router.top", router.get("top")),
        )
        if moe.top > moe.experts:
            raise ConfigError(f"{where}.mlp.router: top={moe.top} is more than the {moe.experts} experts there are")
        fields["moe"] = moe
    return FigosunLayer(**fields)


def figosun_spec(cfg: FigosunConfig) -> ModelSpec:
    norm = {"kind": "rms_norm", "hidden_size": cfg.width, "eps": cfg.norm_eps, "name": ""}
    names = {
        "mixer_norm": "norm1", "mixer_output_norm": "norm1b", "mixer_conv": "canon1", "mixer_gate": "rg1", "mixer": "mix.",
        "ffn_norm": "norm2", "ffn_output_norm": "norm2b", "ffn_conv": "canon2", "ffn_gate": "rg2", "feed_forward": "mlp.",
    }
    layers: list[LayerSpec] = []
    place: dict[int, int] = {}  # config layer that owns tensors -> index into `layers`
    for i, layer in enumerate(cfg.layers):
        if cfg.owners[i] != i:
            continue
        mixer = {
            "kind": "latent_attention", "hidden_size": cfg.width, "num_heads": layer.heads, "head_dim": layer.dim,
            "rot_dim": layer.rot_dim, "v_head_dim": layer.vdim, "kv_rank": layer.kv_rank, "scale": layer.scale,
            "norm_eps": cfg.norm_eps, "output_gate": True,
            # exact_frequencies: base^(-2i/dims) evaluated in 64-bit before it becomes the float32 table
            "position": {"kind": "rotary", "head_dim": layer.rot_dim, "theta": layer.rot_base, "rotary_dim": layer.rot_dim,
                         "interleaved": True, "exact_frequencies": True},
        }
        feed_forward = None
        if layer.moe is not None:
            feed_forward = {
                "kind": "routed_experts", "hidden_size": cfg.width, "intermediate_size": layer.moe.ff, "experts": layer.moe.experts,
                "top": layer.moe.top, "correction": False, "scores": "logistic", "weight_on": "input", "activation": "squared_relu",
            }
        place[i] = len(layers)
        layers.append(LayerSpec(prefix=f"l{i}.", block={
            "kind": "sandwich", "norm": norm, "mixer": mixer, "feed_forward": feed_forward, "hidden_size": cfg.width,
            "gated": True, "conv_taps": cfg.taps, "names": names,
        }))
    return ModelSpec(
        vocab_size=cfg.vocab,
        hidden_size=cfg.width,
        layers=layers,
        order=[LayerCall(place[owner]) for owner in cfg.owners],
        final_norm={**norm, "name": "norm"},
        final_norm_prefix="final.",
        embedding={"kind": "scaled_embedding", "vocab_size": cfg.vocab, "hidden_size": cfg.width, "name": "embed",
                   "scale": cfg.embedding_scale},
        head={"kind": "linear_head", "vocab_size": cfg.vocab, "hidden_size": cfg.width, "name": "head", "tied": True},
    )


FIGOSUN = ARCHITECTURES.register(NAME, Architecture(name=NAME, parse_config=FigosunConfig.from_dict, build_spec=figosun_spec))
