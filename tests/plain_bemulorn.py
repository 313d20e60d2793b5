"""Bemulorn, the plain way: NumPy float64, one function per mechanism, loops over tokens.

The yardstick the engine's Bemulorn is measured against.  It shares no code with the package:
it reads the raw config.json keys itself, keeps no cache (every call sees a whole sequence)
and evaluates every sum in 64-bit.

Notation: `x` is the stream [T, W]; `h` what the layer's one norm makes of it; `p`, `i`, `j`
positions counted from 0.

`store` (default: nothing) is applied to every tensor an engine would keep in its compute dtype
(projections, activations, sublayer outputs, cached rows; never the stream or anything inside a
softmax, a norm or a router).  With `bf16_round` the model shows how far bfloat16 storage alone,
with exact arithmetic between, moves the logits: the yardstick of the bfloat16 tests.
"""

from __future__ import annotations

import math

import numpy as np


def keep(a):
    return a


def f32_round(a):
    return np.asarray(a, dtype=np.float32).astype(np.float64)


def bf16_round(a: np.ndarray) -> np.ndarray:
    import torch

    return torch.from_numpy(np.ascontiguousarray(a, dtype=np.float32)).bfloat16().double().numpy()


def logistic(z):
    return 1.0 / (1.0 + np.exp(-z))


def rms_norm(x: np.ndarray, weight: np.ndarray, eps: float) -> np.ndarray:
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * weight


# np.float32 here makes the angles the way a float32 engine makes them (frequency rounded to float32, then
# the product with the position rounded to float32): a yardstick for float32 engines has to know that
ANGLE_TYPE = np.float64


def frequencies(rot: dict) -> tuple[list[float], float]:
    """Radians a position for every rotated pair, and the factor of cosines and sines.  With
    `scaling` pairs that turn at least `fast` times within `original` positions keep their frequency, pairs
    that turn at most `slow` times have it divided by `factor`, and those between get a blend
    that is linear in the pair's number."""
    dims, base = rot["dims"], rot["base"]
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    scaling = rot.get("scaling")
    if scaling is None:
        return plain, 1.0

    def pair_that_turns(times):
        return dims * math.log(scaling["original"] / (2.0 * math.pi * times)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_that_turns(scaling["fast"])), 0)
    hi = min(math.ceil(pair_that_turns(scaling["slow"])), dims - 1)
    blended = []
    for i, f in enumerate(plain):
        stretched = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        blended.append(f / scaling["factor"] * stretched + f * (1.0 - stretched))
    return blended, 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_halves(rows: np.ndarray, position: int, rot: dict, turns=None) -> np.ndarray:
    """Turn the first `dims` entries of every row of `rows` [n, d], entry i with entry i + dims/2; the rest
    pass.  `turns`: what `frequencies(rot)` gives, if the caller has it."""
    speeds, amplitude = frequencies(rot) if turns is None else turns
    out = np.array(rows, dtype=np.float64)
    half = rot["dims"] // 2
    for i, f in enumerate(speeds):
        angle = float(ANGLE_TYPE(position) * ANGLE_TYPE(f))
        c, s = math.cos(angle) * amplitude, math.sin(angle) * amplitude
        out[:, i] = rows[:, i] * c - rows[:, i + half] * s
        out[:, i + half] = rows[:, i + half] * c + rows[:, i] * s
    return out


def rotate_all(heads: np.ndarray, rot: dict | None, store=keep) -> np.ndarray:
    """Heads [T, n, d] of positions 0 .. T - 1, each turned by its position (no rotation: as they are)."""
    if rot is None:
        return heads
    turns = frequencies(rot)
    return store(np.stack([rotate_halves(heads[t], t, rot, turns) for t in range(heads.shape[0])]))


def embed(tokens, weights: dict, scale: float) -> np.ndarray:
    """Scaled token rows plus the row of each position."""
    return np.stack([weights["embed"][t] * scale + weights["pos"][p] for p, t in enumerate(tokens)]).astype(np.float64)


def visible(i: int, mask: dict | None) -> range:
    """Positions that position i sees: those up to i inside its own stretch of `size` positions."""
    return range(0 if mask is None else i - i % mask["size"], i + 1)


def softmax_plus_one(scores: np.ndarray) -> np.ndarray:
    """exp(s_j) / (1 + sum exp(s))."""
    top = max(float(scores.max()), 0.0)
    e = np.exp(scores - top)
    return e / (math.exp(-top) + e.sum())


def keys_and_values(h: np.ndarray, w: dict, m: dict, store=keep) -> tuple[np.ndarray, np.ndarray]:
    """What a layer with projections of its own caches: rotated keys [T, G, d], values [T, G, dv]."""
    T, G = h.shape[0], m["kv_heads"]
    k = store(h @ w["k"].T + w["k.b"]).reshape(T, G, m["dim"])
    v = store(h @ w["v"].T + w["v.b"]).reshape(T, G, m["vdim"])
    return rotate_all(k, m.get("rot"), store), v


def attention(h: np.ndarray, w: dict, m: dict, keys: np.ndarray, values: np.ndarray, store=keep) -> np.ndarray:
    """Queries of h over the keys and values given (the layer's own or an earlier layer's)."""
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate_all(store(h @ w["q"].T + w["q.b"]).reshape(T, H, d), m.get("rot"), store)
    gate = logistic(store(h @ w["g"].T))  # [T, H]
    out = np.zeros((T, H, dv))
    for a in range(H):
        g = a // (H // G)
        for i in range(T):
            js = visible(i, m.get("mask"))
            p = softmax_plus_one(keys[js.start:js.stop, g] @ q[i, a] * m["scale"])
            out[i, a] = p @ values[js.start:js.stop, g] * gate[i, a]
    return store(store(out.reshape(T, H * dv)) @ w["o"].T)


def clamped_feed_forward(h: np.ndarray, w: dict, limit: float, store=keep) -> np.ndarray:
    g = np.minimum(store(h @ w["gate"].T), limit)
    u = np.clip(store(h @ w["up"].T), -limit, limit)
    return store(store(g * logistic(1.702 * g) * (u + 1.0)) @ w["down"].T)


def silu_feed_forward(h: np.ndarray, w: dict, store=keep) -> np.ndarray:
    z = store(h @ w["gate"].T)
    return store(store(z * logistic(z) * store(h @ w["up"].T)) @ w["down"].T)


# a list here collects, for every token of every routed layer, how far the last chosen expert's logit lies
# above the best one left out (a test can then keep to inputs whose choices no rounding turns)
CHOICE_MARGINS: list | None = None


def routed_feed_forward(h: np.ndarray, w: dict, mlp: dict, store=keep) -> np.ndarray:
    """Each token's `top` experts by biased logit, weighted by the softmax over the chosen logits alone;
    a shared expert, if there is one, is added as it is."""
    router = mlp["router"]
    top = router["top"]
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        z = w["router"] @ h[t] + w["router.b"]
        ranked = np.argsort(-z, kind="stable")
        if CHOICE_MARGINS is not None and top < len(ranked):
            CHOICE_MARGINS.append(float(z[ranked[top - 1]] - z[ranked[top]]))
        chosen = ranked[:top]
        share = np.exp(z[chosen] - z[chosen].max())
        share = share / share.sum()
        for part, e in zip(share, chosen):
            sub = {name: w[f"e{e}.{name}"] for name in ("gate", "up", "down")}
            out[t] += part * silu_feed_forward(h[t:t + 1], sub, store)[0]
    if mlp.get("shared") is not None:
        out += silu_feed_forward(h, {name: w[f"shared.{name}"] for name in ("gate", "up", "down")}, store)
    return store(out)


def split_weights(weights: dict, prefix: str) -> dict:
    return {name[len(prefix):]: np.asarray(value, dtype=np.float64) for name, value in weights.items() if name.startswith(prefix)}


def forward(config: dict, weights: dict, tokens, store=keep, layers_out: list | None = None) -> np.ndarray:
    """The stream after the last layer, [T, W]; `layers_out` collects it after every layer."""
    x = embed(list(tokens), weights, config["embedding"]["scale"])
    cached: dict[int, tuple[np.ndarray, np.ndarray]] = {}
    for n, layer in enumerate(config["layers"]):
        m, mix = layer["mixer"], split_weights(weights, f"l{n}.mix.")
        h = store(rms_norm(x, np.asarray(weights[f"l{n}.norm1"], dtype=np.float64), config["norm"]["eps"]))
        source = m.get("kv_from")
        if source is None:
            cached[n] = keys_and_values(h, mix, m, store)
        y = attention(h, mix, m, *cached[n if source is None else source], store)
        mlp = layer.get("mlp")
        if mlp is not None:
            own = split_weights(weights, f"l{n}.mlp.")
            y = y + (clamped_feed_forward(h, own, mlp["limit"], store) if mlp["kind"] == "dense" else routed_feed_forward(h, own, mlp, store))
        x = x + y
        if layers_out is not None:
            layers_out.append(x.copy())
    return x


def logits(config: dict, weights: dict, tokens, store=keep, layers_out: list | None = None) -> np.ndarray:
    x = forward(config, weights, tokens, store, layers_out)
    h = store(rms_norm(x, np.asarray(weights["final.norm"], dtype=np.float64), config["norm"]["eps"]))
    return h @ np.asarray(weights["head"], dtype=np.float64).T * config["logit_scale"]


def greedy(row: np.ndarray) -> int:
    return int(np.argmax(row))
