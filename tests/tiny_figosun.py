"""Tiny Figosun configurations, weights and model folders for the tests.

The configurations differ in every size and constant and in the order of layers: layers with and
without a feed-forward; tensors shared once, twice and through a chain of layers; one to five taps;
one head, several, more than a wave's rows; value heads narrower and wider than query heads; latents
that the matrix-core kernels take (in general and in their exact forms) and latents they do not; one
expert of one, one of several, several, all; sizes that no vector width divides.  Weights are made
with NumPy and rounded to bfloat16, so both engines and the plain model read the same numbers.
"""

from __future__ import annotations

import json
from pathlib import Path

import numpy as np
import torch
from safetensors.torch import save_file


def moe(ff, experts, top):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def latent(heads, dim, rot_dim, vdim, kv_rank, scale, base, mlp=None):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
                      "rot": {"base": base, "dims": rot_dim}},
            "mlp": mlp}


def again(layers, of):
    """A layer that runs with the tensors of layer `of`."""
    return {**layers[of], "weights_of": of}


def config(vocab, width, layers, *, eps, taps, scale):
    return {"architecture": "Figosun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "canon": {"taps": taps},
            "embedding": {"scale": scale}, "layers": layers}


# a layer without feed-forward; two layers run with the first one's tensors; value heads wider than query
# heads; a latent the matrix-core kernel does not take
_A = [latent(4, 10, 6, 24, 22, 0.5, 50.0, moe(48, 6, 2)), latent(3, 8, 8, 6, 14, 0.6, 1000.0)]
_A += [again(_A, 0), latent(8, 12, 4, 12, 34, 0.4, 7.0, moe(32, 4, 1)), again(_A, 0)]
TINY_A, TINY_A_BLOCK = config(150, 64, _A, eps=1e-5, taps=4, scale=3.0), 16
# sizes nothing divides; two taps; all experts chosen; a chain of layers that name one another
_B = [latent(5, 6, 2, 10, 18, 0.9, 20.0, moe(26, 3, 3)), latent(2, 4, 4, 6, 10, 1.0, 100.0, moe(22, 5, 4))]
_B += [again(_B, 1)]
_B += [again(_B, 2), again(_B, 0)]
TINY_B, TINY_B_BLOCK = config(131, 90, _B, eps=3e-6, taps=2, scale=1.0), 8
# sizes at which the fast bfloat16 paths run (weight-streaming products, whole vector loads, expert tiles, latent
# heads that the matrix cores take when a prompt comes whole: 32 + 32 and 64 + 64)
_C = [latent(4, 32, 32, 48, 80, 0.2, 10000.0, moe(128, 8, 2)), latent(2, 64, 64, 128, 128, 0.15, 500000.0, moe(64, 16, 4))]
_C += [again(_C, 0), latent(6, 16, 16, 32, 48, 0.25, 300.0)]
TINY_C, TINY_C_BLOCK = config(300, 256, _C, eps=2e-6, taps=3, scale=2.0), 16
# one tap (no state but pages), one head, one expert of one; pages of 4
_D = [latent(1, 8, 4, 8, 12, 0.7, 100.0, moe(16, 1, 1)), latent(2, 8, 2, 12, 16, 0.8, 30.0)]
_D += [again(_D, 1)]
TINY_D, TINY_D_BLOCK = config(97, 48, _D, eps=1e-6, taps=1, scale=0.5), 4
# latents of the sizes the matrix-core kernel has exact forms for, and one between; more heads than a wave has rows; five taps
_E = [latent(3, 16, 64, 16, 512, 0.2, 10000.0, moe(64, 4, 2)), latent(17, 16, 32, 8, 256, 0.25, 1000.0), latent(20, 8, 24, 16, 304, 0.3, 50.0)]
TINY_E, TINY_E_BLOCK = config(120, 128, _E, eps=1e-6, taps=5, scale=1.5), 16

CONFIGS = {"A": (TINY_A, TINY_A_BLOCK), "B": (TINY_B, TINY_B_BLOCK), "C": (TINY_C, TINY_C_BLOCK), "D": (TINY_D, TINY_D_BLOCK),
           "E": (TINY_E, TINY_E_BLOCK)}


def bf16_round(values: np.ndarray) -> np.ndarray:
    return torch.from_numpy(np.ascontiguousarray(values, dtype=np.float32)).bfloat16().float().numpy()


def tensor_shapes(cfg: dict) -> dict[str, tuple[int, ...]]:
    w, v, taps = cfg["width"], cfg["vocab"], cfg["canon"]["taps"]
    shapes: dict[str, tuple[int, ...]] = {"embed": (v, w), "final.norm": (w,)}
    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p, m, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        for q in ("1", "2") if mlp is not None else ("1",):
            shapes.update({p + "norm" + q: (w,), p + f"norm{q}b": (w,), p + "canon" + q: (w, taps), p + "rg" + q: (w, w), p + f"rg{q}.b": (w,)})
        shapes.update({p + "mix.q": (m["heads"] * (m["dim"] + m["rot_dim"]), w), p + "mix.dkv": (m["kv_rank"] + m["rot_dim"], w),
                       p + "mix.dkv.norm": (m["kv_rank"],), p + "mix.uk": (m["heads"] * m["dim"], m["kv_rank"]),
                       p + "mix.uv": (m["heads"] * m["vdim"], m["kv_rank"]), p + "mix.g": (m["heads"] * m["vdim"], w),
                       p + "mix.o": (w, m["heads"] * m["vdim"])})
        if mlp is None:
            continue
        ff = mlp["expert"]["ff"]
        shapes[p + "mlp.router"] = (mlp["router"]["experts"], w)
        for e in range(mlp["router"]["experts"]):
            shapes.update({p + f"mlp.e{e}.up": (ff, w), p + f"mlp.e{e}.down": (w, ff)})
    return shapes


def make_weights(cfg: dict, seed: int, steady_choice: bool = False) -> dict[str, np.ndarray]:
    """Activations of order one everywhere; norm weights spread widely and convolutions and gate biases of order one
    (one left out shows), attention sharp enough that single keys matter, routers with rows of order several.

    `steady_choice`: the first column of the stream is large and the same for every token (one column of the
    embedding is constant, no convolution on it), and the routers' first column sets their logits far apart, so every token
    chooses the same experts (each with the token's own weights).  The stream of a bfloat16 engine differs from
    the exact one by a percent or so after a few layers, and among hundreds of tokens some choice always
    hangs on less than that; a chosen expert that differs is no rounding error.  Whole models in bfloat16 are
    therefore tested with steady choices, and the choice itself where both sides read the same bits: the
    router's kernel alone, in both dtypes, and whole models in the 32-bit engine."""
    rng = np.random.default_rng(seed)
    out: dict[str, np.ndarray] = {}
    for name, shape in sorted(tensor_shapes(cfg).items()):
        leaf = name.split(".", 1)[-1] if name.startswith("l") and name[1].isdigit() else name
        if leaf in ("norm1", "norm2", "final.norm", "mix.dkv.norm"):
            values = rng.uniform(0.5, 1.5, size=shape)
        elif leaf in ("norm1b", "norm2b"):
            values = rng.uniform(0.3, 0.9, size=shape)
        elif leaf in ("canon1", "canon2"):
            values = rng.standard_normal(shape) * 0.4
        elif leaf in ("rg1.b", "rg2.b"):
            values = rng.standard_normal(shape) * 1.5
        elif leaf == "mlp.router":
            values = rng.standard_normal(shape) * 2.0 / np.sqrt(shape[1])
        elif name == "embed":
            values = rng.standard_normal(shape) * 0.4  # (the table is the head too: logits of a few units)
        else:
            values = rng.standard_normal(shape) / np.sqrt(shape[1]) * (2.0 if leaf in ("mix.q", "mix.uk") else 1.0)
        if steady_choice:
            if name == "embed":
                values[:, 0] = 10.0 / cfg["embedding"]["scale"]
            elif leaf in ("norm2",):
                values[0] = 0.25
            elif leaf == "norm1":
                values[0] = 0.1
            elif leaf == "final.norm":
                values[0] = 0.0  # (the table is the head too: its constant column would add one large number to all logits)
            elif leaf in ("norm1b", "norm2b"):
                values[0] = 0.1
            elif leaf in ("canon1", "canon2"):
                values[0] = 0.0
            elif leaf == "mlp.router":
                values *= 0.15
                values[:, 0] = 0.5 - 1.6 * rng.permutation(shape[0])
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
