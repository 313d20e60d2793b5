"""Tiny Bemulorn configurations, weights and model folders for the tests.

The configurations differ in every size and constant and in the order of layers: dense or routed
first; layers without a feed-forward; keys and values shared by two and by three layers, by neighbours and
across others, with chunks equal to and other than their owner's; chunks of one position, smaller than a page,
a page's multiple, none, longer than any prompt; one key/value head, several, as many as query heads; value
heads wider, narrower and as wide as key heads; rotation of a whole head, a part, nothing, with all of a
blend's three ranges, with frequencies left alone, and with one that ends where it begins; experts with and
without a shared one, one chosen, several, all; scales of 1 and others; sizes that no vector width divides.
Weights are made with NumPy and rounded to bfloat16, so both engines and the plain model read the same
numbers.
"""

from __future__ import annotations

import json
from pathlib import Path

import numpy as np
import torch
from safetensors.torch import save_file


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(ff, experts, top, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def rotation(base, dims, scaling=None):
    """`scaling`: (factor, original, fast, slow) or None."""
    rot = {"base": base, "dims": dims}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return rot


def attention(heads, kv_heads, dim, vdim, scale, chunk=None, rot=None, mlp=None, kv_from=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk is not None:
        mixer["mask"] = {"size": chunk}
    if rot is not None:
        mixer["rot"] = rot
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def config(vocab, width, layers, *, eps, scale=1.0, logit_scale=1.0, positions=512):
    return {"architecture": "Bemulorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "logit_scale": logit_scale, "max_positions": positions, "layers": layers}


YARN_A = rotation(300.0, 12, (4.0, 64, 8.0, 1.0))
# routed first; a reader with another chunk than its owner's (so nothing is given back) and one behind a layer that
# owns keys too; a layer without feed-forward; chunks that are no multiple of a page
TINY_A = config(150, 64, [
    attention(4, 2, 16, 24, 0.5, chunk=20, rot=YARN_A, mlp=moe(48, 6, 2, shared=40)),
    attention(6, 2, 16, 24, 0.4, chunk=33, rot=YARN_A, mlp=dense(80, 1.5), kv_from=0),
    attention(4, 1, 24, 8, 0.35, chunk=50, rot=rotation(50.0, 24, (2.5, 32, 3.0, 0.5))),
    attention(8, 2, 16, 24, 0.5, chunk=20, rot=YARN_A, mlp=moe(32, 4, 1), kv_from=0),
    attention(4, 1, 24, 8, 0.3, chunk=50, rot=rotation(50.0, 24, (2.5, 32, 3.0, 0.5)), mlp=dense(32, 4.0), kv_from=2),
], eps=1e-5, scale=2.5, logit_scale=1.75)
TINY_A_BLOCK = 16
# sizes nothing divides; one chunk longer than any prompt and one layer without; all experts chosen; no shared
# expert; as many key/value heads as query heads and a single one; no rotation at all in one layer; page size 8
TINY_B = config(131, 90, [
    attention(3, 3, 10, 6, 0.7, rot=rotation(11.0, 6), mlp=moe(26, 3, 3)),
    attention(5, 1, 6, 10, 0.8, chunk=400, rot=rotation(1000.0, 6, (9.0, 20, 30.0, 2.0)), mlp=dense(70, 0.8)),
    attention(2, 1, 6, 10, 0.9, chunk=7, rot=rotation(1000.0, 6, (9.0, 20, 30.0, 2.0)), mlp=moe(22, 5, 4, shared=30), kv_from=1),
    attention(7, 7, 4, 14, 0.6, chunk=11),
], eps=3e-6, scale=1.0, logit_scale=0.6)
TINY_B_BLOCK = 8
# sizes at which the fast bfloat16 paths run: weight-streaming products with everything folded in, value heads of
# their own width on the matrix cores (64 and 112 beside 64; 48 beside 96), the tiles of routed experts
YARN_C = rotation(10000.0, 32, (8.0, 128, 32.0, 1.0))
TINY_C = config(300, 192, [
    attention(6, 2, 64, 112, 0.2, chunk=48, rot=YARN_C, mlp=dense(320, 2.5)),
    attention(4, 1, 96, 48, 0.15, chunk=64, rot=rotation(500000.0, 96), mlp=moe(64, 16, 4, shared=128)),
    attention(12, 2, 64, 112, 0.22, chunk=48, rot=YARN_C, mlp=moe(128, 8, 2), kv_from=0),
    attention(8, 1, 96, 48, 0.15, chunk=64, rot=rotation(500000.0, 96), mlp=dense(256, 7.0), kv_from=1),
], eps=2e-6, scale=3.5, logit_scale=1.25)
TINY_C_BLOCK = 16
# chunks beside page borders: a page of 4 with chunks of 4, 5, 8, 3 and 1
TINY_D = config(97, 48, [
    attention(2, 1, 8, 8, 1.0, chunk=4, rot=rotation(20.0, 4), mlp=dense(16, 3.0)),
    attention(4, 2, 8, 6, 0.9, chunk=5, rot=rotation(100.0, 8, (3.0, 10, 2.0, 1.0))),
    attention(2, 2, 12, 12, 0.8, chunk=8, mlp=moe(16, 2, 1, shared=8)),
    attention(4, 2, 8, 6, 1.1, chunk=3, rot=rotation(100.0, 8, (3.0, 10, 2.0, 1.0)), kv_from=1),
    attention(3, 1, 6, 8, 1.0, chunk=1, mlp=dense(24, 2.0)),
], eps=1e-6, scale=0.75, logit_scale=3.0)
TINY_D_BLOCK = 4
# values as wide as keys on the matrix cores; one head; dense layers alone, so that a decode step hands products and
# norm factors from layer to layer
TINY_E = config(210, 128, [
    attention(4, 4, 32, 32, 0.3, chunk=96, rot=rotation(700.0, 16, (2.0, 48, 4.0, 1.0)), mlp=dense(192, 1.2)),
    attention(8, 4, 32, 32, 0.3, chunk=96, rot=rotation(700.0, 16, (2.0, 48, 4.0, 1.0)), mlp=dense(64, 2.2), kv_from=0),
    attention(1, 1, 128, 128, 0.09, chunk=80, rot=rotation(100.0, 128), mlp=dense(128, 1.0)),
], eps=1e-4, scale=1.5, logit_scale=1.0)
TINY_E_BLOCK = 16

CONFIGS = {"A": (TINY_A, TINY_A_BLOCK), "B": (TINY_B, TINY_B_BLOCK), "C": (TINY_C, TINY_C_BLOCK), "D": (TINY_D, TINY_D_BLOCK),
           "E": (TINY_E, TINY_E_BLOCK)}


def bf16_round(values: np.ndarray) -> np.ndarray:
    return torch.from_numpy(np.ascontiguousarray(values, dtype=np.float32)).bfloat16().float().numpy()


def tensor_shapes(cfg: dict) -> dict[str, tuple[int, ...]]:
    w, v = cfg["width"], cfg["vocab"]
    shapes: dict[str, tuple[int, ...]] = {"embed": (v, w), "pos": (cfg["max_positions"], w), "final.norm": (w,), "head": (v, w)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        q = m["heads"] * m["dim"]
        shapes.update({p + "norm1": (w,), p + "mix.q": (q, w), p + "mix.q.b": (q,), p + "mix.g": (m["heads"], w),
                       p + "mix.o": (w, m["heads"] * m["vdim"])})
        if m.get("kv_from") is None:
            for name, rows in (("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                shapes.update({p + "mix." + name: (rows, w), p + "mix." + name + ".b": (rows,)})
        mlp = layer["mlp"]
        if mlp is None:
            continue
        gated = {"": mlp["ff"]} if mlp["kind"] == "dense" else {f"e{e}.": mlp["expert"]["ff"] for e in range(mlp["router"]["experts"])}
        if mlp["kind"] == "moe":
            shapes.update({p + "mlp.router": (mlp["router"]["experts"], w), p + "mlp.router.b": (mlp["router"]["experts"],)})
            if mlp.get("shared"):
                gated["shared."] = mlp["shared"]["ff"]
        for sub, ff in gated.items():
            shapes.update({p + f"mlp.{sub}gate": (ff, w), p + f"mlp.{sub}up": (ff, w), p + f"mlp.{sub}down": (w, ff)})
    return shapes


def make_weights(cfg: dict, seed: int, steady_choice: bool = False) -> dict[str, np.ndarray]:
    """Activations of order one everywhere: biases of order a half, gates and routers with rows of order two, so
    that each shows where it is left out; products into a clamped feed-forward large enough to be clamped.

    `steady_choice`: every token chooses the same experts (each with the token's own weights): as many as are
    chosen have a bias far above the rest.  The stream of a bfloat16 engine differs from the exact one by a
    percent or so, which moves a token's logits by several hundredths, and among hundreds of tokens some choice
    always hangs on less than that; a chosen expert that differs is no rounding error.  Whole models in bfloat16
    are therefore tested with steady choices, and the choice itself where the inputs are the same bits on both
    sides: the router's kernels alone, and whole models in the 32-bit engine."""
    rng = np.random.default_rng(seed)
    out: dict[str, np.ndarray] = {}
    for name, shape in sorted(tensor_shapes(cfg).items()):
        leaf = name.split(".", 1)[-1] if name.startswith("l") and name[1].isdigit() else name
        if leaf in ("norm1", "final.norm"):
            values = rng.uniform(0.5, 1.5, size=shape)
        elif leaf in ("mix.q.b", "mix.k.b", "mix.v.b"):
            values = rng.standard_normal(shape) * 0.5
        elif leaf == "mlp.router.b":
            values = rng.standard_normal(shape) * 0.7
            if steady_choice:
                top = cfg["layers"][int(name[1:name.index(".")])]["mlp"]["router"]["top"]
                values = np.where(rng.permutation(shape[0]) < top, 6.0, 0.0) + values * 0.1
        elif leaf == "mlp.router":
            values = rng.standard_normal(shape) * (0.5 if steady_choice else 2.0) / np.sqrt(shape[1])
        elif leaf == "mix.g":
            values = rng.standard_normal(shape) * 2.0 / np.sqrt(shape[1])
        elif name in ("embed", "pos"):
            values = rng.standard_normal(shape) * 0.6
        else:
            values = rng.standard_normal(shape) / np.sqrt(shape[1]) * (1.5 if leaf in ("mix.q", "mix.k", "mlp.gate", "mlp.up") else 1.0)
        out[name] = bf16_round(np.asarray(values, dtype=np.float32)).reshape(shape)
    return out


def write_model_dir(path: Path, cfg: dict, weights: dict[str, np.ndarray], dtype=torch.bfloat16) -> Path:
    path = Path(path)
    path.mkdir(parents=True, exist_ok=True)
    with (path / "config.json").open("w") as handle:
        json.dump(cfg, handle)
    tensors = {k: torch.from_numpy(np.ascontiguousarray(v, dtype=np.float32)).reshape(v.shape).to(dtype) for k, v in weights.items()}
    save_file(tensors, str(path / "model.safetensors"))
    return path


def random_tokens(cfg: dict, length: int, seed: int) -> list[int]:
    return np.random.default_rng(seed).integers(0, cfg["vocab"], size=length).tolist()
