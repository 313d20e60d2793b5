"""Rotary position encoding: the inverse-frequency table and how dims are paired.

`inv_freq = theta^(-2j/D)` in float32 (models/blocks/rope.py:343-346 of the
reference), optionally rescaled the llama3 way (rope.py:200-225).  The table
stays float32 whatever the compute dtype (rope.py:368-390), and the angles
`position * inv_freq` and their cos/sin are float32 too.

A mixer asks this part for the cos/sin tables of a step (`rotary(ctx)`); they are
computed once per step and shared by all layers that use the same encoding.
"""

from __future__ import annotations

import math

import torch

from mini_infer_amd import ops
from mini_infer_amd.parts.base import PositionEncoding, RotaryTables, StepContext
from mini_infer_amd.registry import register_position_encoding


def default_inv_freq(rotary_dim: int, theta: float) -> torch.Tensor:
    exponent = torch.arange(0, rotary_dim, 2, dtype=torch.float32) / rotary_dim
    return 1.0 / (theta**exponent)


def exact_inv_freq(rotary_dim: int, theta: float, dtype: torch.dtype = torch.float32) -> torch.Tensor:
    """theta^(-2j/D) evaluated in 64-bit and rounded to float32 once (`default_inv_freq` makes
    the same table in float32 arithmetic, as the reference does, and is a last bit or two off).
    `dtype=torch.float64`: not rounded yet, for a rescaling that is to be exact as well."""
    exponent = torch.arange(0, rotary_dim, 2, dtype=torch.float64) / rotary_dim
    return torch.pow(torch.tensor(float(theta), dtype=torch.float64), -exponent).to(dtype)


def llama3_inv_freq(
    inv_freq: torch.Tensor,
    factor: float,
    low_freq_factor: float,
    high_freq_factor: float,
    original_max_position_embeddings: int,
) -> torch.Tensor:
    """Long wavelengths divided by `factor`, short ones kept, the band between blended."""
    old_len = original_max_position_embeddings
    low_wavelen = old_len / low_freq_factor
    high_wavelen = old_len / high_freq_factor
    wavelen = 2 * math.pi / inv_freq
    scaled = torch.where(wavelen > low_wavelen, inv_freq / factor, inv_freq)
    smooth = (old_len / wavelen - low_freq_factor) / (high_freq_factor - low_freq_factor)
    smoothed = (1 - smooth) * scaled / factor + smooth * scaled
    medium = ~(wavelen < high_wavelen) & ~(wavelen > low_wavelen)
    return torch.where(medium, smoothed, scaled)


def yarn_inv_freq(inv_freq: torch.Tensor, theta: float, factor: float, original: float, fast: float, slow: float) -> torch.Tensor:
    """Frequencies rescaled by how often a pair turns within `original` positions: pairs that turn `fast` times or
    more keep theirs, pairs that turn `slow` times or less have it divided by `factor`, and in between the two are
    blended along the pair's number (whole numbers mark the ends of the blend)."""
    pairs = inv_freq.numel()
    dims = 2 * pairs

    def pair_turning(times: float) -> float:
        return dims * math.log(original / (2 * math.pi * times)) / (2 * math.log(theta))

    first = max(math.floor(pair_turning(fast)), 0)
    last = min(math.ceil(pair_turning(slow)), dims - 1)
    blend = ((torch.arange(pairs, dtype=torch.float64) - first) / max(last - first, 0.001)).clamp(0.0, 1.0).to(inv_freq.dtype)
    return inv_freq / factor * blend + inv_freq * (1 - blend)


def yarn_amplitude(factor: float) -> float:
    """What cosines and sines are multiplied by beside `yarn_inv_freq`."""
    return 0.1 * math.log(factor) + 1.0


class RotaryPosition(PositionEncoding):
    """Rotation of the first `rotary_dim` dims of each head.

    `interleaved=False` pairs dim j with j + rotary_dim/2 (the Llama way,
    rope.py:411-416); `interleaved=True` pairs 2j with 2j+1.  `yarn` = {"factor", "original", "fast", "slow"}:
    frequencies rescaled by `yarn_inv_freq`, cosines and sines by `yarn_amplitude`.
    """

    def __init__(
        self,
        head_dim: int,
        theta: float,
        dtype: torch.dtype,
        device,
        *,
        rotary_dim: int | None = None,
        interleaved: bool = False,
        llama3: dict | None = None,
        exact_frequencies: bool = False,
        yarn: dict | None = None,
    ) -> None:
        super().__init__(dtype, device)
        self.head_dim = head_dim
        self.rotary_dim = head_dim if rotary_dim is None else int(rotary_dim)
        if self.rotary_dim % 2 != 0 or not 0 < self.rotary_dim <= head_dim:
            raise ValueError(f"rotary_dim={self.rotary_dim} must be even and within head_dim={head_dim}")
        self.interleaved = bool(interleaved)
        if exact_frequencies:  # (the rescaling too in 64-bit; one rounding at the end)
            table = exact_inv_freq(self.rotary_dim, float(theta), torch.float64)
        else:
            table = default_inv_freq(self.rotary_dim, float(theta))
        if llama3 is not None:
            table = llama3_inv_freq(
                table,
                float(llama3["factor"]),
                float(llama3["low_freq_factor"]),
                float(llama3["high_freq_factor"]),
                int(llama3["original_max_position_embeddings"]),
            )
        self.amplitude = 1.0
        if yarn is not None:
            if llama3 is not None:
                raise ValueError("rotary frequencies are rescaled one way, not two")
            table = yarn_inv_freq(table, float(theta), float(yarn["factor"]), float(yarn["original"]), float(yarn["fast"]), float(yarn["slow"]))
            self.amplitude = yarn_amplitude(float(yarn["factor"]))
        self.inv_freq_host = table.to(torch.float32)
        self._inv_freq_device: torch.Tensor | None = None

    @property
    def inv_freq(self) -> torch.Tensor:
        if self._inv_freq_device is None:
            self._inv_freq_device = self.inv_freq_host.to(self.device).contiguous()
        return self._inv_freq_device

    def tables(self, ctx: StepContext) -> tuple[torch.Tensor, torch.Tensor]:
        """cos, sin [T, rotary_dim/2] float32 for this step's positions (made once a step)."""
        key = ("rotary_tables", id(self))
        if key not in ctx.shared:
            ctx.shared[key] = ops.rope_table(ctx.positions, self.inv_freq, self.amplitude)
        return ctx.shared[key]

    def rotary_layout(self) -> tuple[int, bool]:
        return self.rotary_dim, self.interleaved

    def rotary(self, ctx: StepContext) -> RotaryTables:
        cos, sin = self.tables(ctx)
        return RotaryTables(cos, sin, self.rotary_dim, self.interleaved)


@register_position_encoding("rotary")
def build_rotary(desc: dict, dtype: torch.dtype, device, shared: dict | None = None) -> RotaryPosition:
    return RotaryPosition(
        int(desc["head_dim"]),
        float(desc["theta"]),
        dtype,
        device,
        rotary_dim=desc.get("rotary_dim"),
        interleaved=bool(desc.get("interleaved", False)),
        llama3=desc.get("llama3"),
        exact_frequencies=bool(desc.get("exact_frequencies", False)),
        yarn=desc.get("yarn"),
    )


class DistanceSlopes(PositionEncoding):
    """No rotation: positions enter the scores as a penalty linear in the distance, `slope_h * (i - j)`
    taken off the score of query head h at position i for the key at position j, with slopes in a
    geometric row, `slope_h = 2^(-total * (h + 1) / heads)` for h = 0 .. heads - 1."""

    graph_safe = True

    def __init__(self, total_exponent: float, dtype: torch.dtype, device) -> None:
        super().__init__(dtype, device)
        self.total_exponent = float(total_exponent)

    def score_slopes(self, num_heads: int) -> torch.Tensor:
        heads = torch.arange(1, num_heads + 1, dtype=torch.float64)
        return torch.pow(2.0, -self.total_exponent * heads / num_heads).to(torch.float32).to(self.device).contiguous()


@register_position_encoding("distance_slopes")
def build_distance_slopes(desc: dict, dtype: torch.dtype, device, shared: dict | None = None) -> DistanceSlopes:
    return DistanceSlopes(float(desc.get("total_exponent", 8.0)), dtype, device)
