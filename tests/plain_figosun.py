"""Figosun, the plain way: NumPy float64, one function per mechanism.

The yardstick the engine's Figosun is measured against.  It shares no code with the package: it
reads the raw config.json keys itself, keeps no cache and no state (every call sees a whole
sequence) and evaluates every sum in 64-bit.

Notation: `x` is the stream [T, W]; `h` what a sublayer's norm made of it; `i`, `j`, `t` positions
counted from 0.

`store` (default: nothing) is applied to every tensor an engine would keep in its compute dtype
(norm outputs, projections, activations, sublayer outputs, cached rows, logits; never the stream or
anything inside a softmax, a norm or a router).  With `bf16_round` the model shows how far bfloat16
storage alone, with exact arithmetic between, moves the logits: the yardstick of the bfloat16 tests.
"""

from __future__ import annotations

import numpy as np


def keep(a):
    return a


def bf16_round(a: np.ndarray) -> np.ndarray:
    import torch

    return torch.from_numpy(np.ascontiguousarray(a, dtype=np.float32)).bfloat16().double().numpy()


def f32_round(a: np.ndarray) -> np.ndarray:
    return np.asarray(a, dtype=np.float32).astype(np.float64)


def rms_norm(x: np.ndarray, weight: np.ndarray, eps: float) -> np.ndarray:
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * weight


def logistic(z):
    return 1.0 / (1.0 + np.exp(-z))


def squared_relu(z):
    return np.maximum(z, 0.0) ** 2


# np.float32 here makes the angles the way a float32 engine makes them (frequency rounded to float32, then
# the product with the position rounded to float32)
ANGLE_TYPE = np.float64


def rotate_pairs(v: np.ndarray, position: int, base: float, dims: int) -> np.ndarray:
    """Rotate the first `dims` entries of the last axis of `v`, entry 2i with entry 2i+1, by the angle
    position * base^(-2i/dims)."""
    out = np.array(v, dtype=np.float64)
    for i in range(dims // 2):
        angle = float(ANGLE_TYPE(position) * ANGLE_TYPE(base ** (-2.0 * i / dims)))
        a, b = np.array(v[..., 2 * i]), np.array(v[..., 2 * i + 1])
        out[..., 2 * i] = a * np.cos(angle) - b * np.sin(angle)
        out[..., 2 * i + 1] = b * np.cos(angle) + a * np.sin(angle)
    return out


def embed(tokens, weights: dict, scale: float) -> np.ndarray:
    return np.stack([weights["embed"][t] for t in tokens]).astype(np.float64) * scale


def causal_conv(h: np.ndarray, taps_weight: np.ndarray) -> np.ndarray:
    """Per channel: sum over the taps, the last one on the current row, of the rows before (zeros
    ahead of the first)."""
    T, taps = h.shape[0], taps_weight.shape[1]
    out = np.zeros_like(h)
    for t in range(T):
        for j in range(taps):
            at = t - (taps - 1) + j
            if at >= 0:
                out[t] += taps_weight[:, j] * h[at]
    return out


def residual_gate(h: np.ndarray, weight: np.ndarray, bias: np.ndarray, store=keep) -> np.ndarray:
    """What a sublayer's result is multiplied with, element by element."""
    return logistic(store(h @ weight.T) + bias)


def latent_attention(h: np.ndarray, w: dict, m: dict, eps: float, store=keep) -> np.ndarray:
    """Keys and values of all heads as maps of one normed latent row per token, beside one rotated key
    part that the heads share; every earlier position is seen; the heads' outputs are gated."""
    T = h.shape[0]
    H, d, r, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    base, dims = m["rot"]["base"], m["rot"]["dims"]
    q = store(h @ w["q"].T).reshape(T, H, d + r)
    down = store(h @ w["dkv"].T)
    c = store(rms_norm(down[:, :rank], w["dkv.norm"], eps))
    shared_key = store(np.stack([rotate_pairs(down[i, rank:], i, base, dims) for i in range(T)]))
    keys = (c @ w["uk"].T).reshape(T, H, d)
    values = (c @ w["uv"].T).reshape(T, H, dv)
    out = np.zeros((T, H, dv))
    for i in range(T):
        q_rot = rotate_pairs(q[i, :, d:], i, base, dims)
        for a in range(H):
            s = (keys[: i + 1, a] @ q[i, a, :d] + shared_key[: i + 1] @ q_rot[a]) * m["scale"]
            p = np.exp(s - s.max())
            out[i, a] = (p / p.sum()) @ values[: i + 1, a]
    gate = logistic(store(h @ w["g"].T))
    return store(store(store(out.reshape(T, H * dv)) * gate) @ w["o"].T)


# a list here collects, for every token of every routed layer, how far the last chosen expert's router
# logit lies above the best one left out (a test can then keep to inputs whose choices no rounding turns)
CHOICE_MARGINS: list | None = None


def routed_feed_forward(h: np.ndarray, w: dict, mlp: dict, store=keep) -> np.ndarray:
    """Each token's `top` experts by score, an expert's score multiplying what it READS."""
    experts, top = mlp["router"]["experts"], mlp["router"]["top"]
    out = np.zeros_like(h)
    logits = h @ w["router"].astype(np.float64).T
    for t in range(h.shape[0]):
        scores = logistic(logits[t])
        ranked = np.argsort(-logits[t], kind="stable")
        if CHOICE_MARGINS is not None and top < experts:
            CHOICE_MARGINS.append(float(logits[t, ranked[top - 1]] - logits[t, ranked[top]]))
        for e in ranked[:top]:
            act = store(squared_relu(w[f"e{e}.up"] @ (scores[e] * h[t])))
            out[t] += store(w[f"e{e}.down"] @ act)
    return store(out)


def split_weights(weights: dict, prefix: str) -> dict:
    return {name[len(prefix):]: np.asarray(value, dtype=np.float64) for name, value in weights.items() if name.startswith(prefix)}


def owner_of(layers: list, n: int) -> int:
    """The layer whose tensors layer n runs with."""
    while layers[n].get("weights_of") is not None:
        n = layers[n]["weights_of"]
    return n


def sublayer(x, w, mark, run, eps, store=keep):
    """x + norm_b( gate(h) * run(h + conv(h)) ),  h = norm(x)."""
    h = store(rms_norm(x, w["norm" + mark], eps))
    u = store(h + causal_conv(h, w["canon" + mark]))
    y = run(u) * residual_gate(h, w["rg" + mark], w["rg" + mark + ".b"], store)
    return x + rms_norm(y, w["norm" + mark + "b"], eps)


def forward(config: dict, weights: dict, tokens, store=keep, layers_out: list | None = None) -> np.ndarray:
    """The stream after the last layer, [T, W]; `layers_out` collects it after every layer."""
    eps = config["norm"]["eps"]
    x = embed(list(tokens), weights, config["embedding"]["scale"])
    for n, layer in enumerate(config["layers"]):
        prefix = f"l{owner_of(config['layers'], n)}."
        w, mix, mlp = (split_weights(weights, prefix + part) for part in ("", "mix.", "mlp."))
        if layer["type"] != "latent_attention":
            raise ValueError(layer["type"])
        x = sublayer(x, w, "1", lambda u: latent_attention(u, mix, layer["mixer"], eps, store), eps, store)
        if layer.get("mlp") is not None:
            x = sublayer(x, w, "2", lambda u: routed_feed_forward(u, mlp, layer["mlp"], store), eps, store)
        if layers_out is not None:
            layers_out.append(x.copy())
    return x


def logits(config: dict, weights: dict, tokens, store=keep, layers_out: list | None = None) -> np.ndarray:
    x = forward(config, weights, tokens, store, layers_out)
    h = store(rms_norm(x, np.asarray(weights["final.norm"], dtype=np.float64), config["norm"]["eps"]))
    return store(h @ np.asarray(weights["embed"], dtype=np.float64).T)


def greedy(row: np.ndarray) -> int:
    return int(np.argmax(row))
