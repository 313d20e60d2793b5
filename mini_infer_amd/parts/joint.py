"""A layer whose sublayers read one norm, with their products made together.

Where a mixer and a gated feed-forward read the same rows h and their results are added up,

    y = W_o mix(W_m h) + W_down act(W_gate h, W_up h),

the two first products are one product with the stacked rows [W_m; W_gate; W_up], and, since
both results are sums, the two last ones are one product with the matrices side by side,

    y = [W_o | W_down] [mix(..); act(..)]

(the sum of the sublayers is then rounded once, not three times).  A layer is two products of
twice the size with the mixer's own work between them: at few rows the weights of a whole layer stream
through two launches, and the first of them ends with everything that follows it row by row
(`ops.layer_in`).  For many rows the vendor library makes both products and the pieces of a very large one are
faster apart, so a prompt takes the parts' own views of the stacked matrices where they are (`apart_in`,
`apart_out`).

What a mixer that joins offers (`Mixer.can_join`): `joint_input` and `joint_output` (its first and
last `Linear`), `joint_layout(ff, limit, slope)` (how the stacked rows lie), `rotation()`,
`forward_projected(columns, ctx, cache, writes_cache, out)` and `forward_layer_in(...)`.  What a
feed-forward that joins offers (`FeedForward.joint_partner`): `gate_up` and `down` (`Linear`s),
`joint_limits`, and `forward_projected(columns, out)`.  Both keep working on their own: their weights become
views of the stacked matrices.
"""

from __future__ import annotations

import torch

from mini_infer_amd import ops
from mini_infer_amd.parts.base import FeedForward, LayerCache, Mixer, StepContext

ROW_STEP = 8  # rows of stacked products and of joined inner rows begin on boundaries of as many elements


# Where bfloat16 products are made apart (bfloat16 only; the 32-bit engine's own product has no such choice).
# The first product, by rows x stacked features, microseconds together / apart at 8B and 1B widths:
#     512 x 34592    147 / 128      1024 x 13088    96 / 108      256 x 34592     83 / 94
#     2048 x 34592   466 / 430      2048 x 11296   255 / 155      2048 x 6176     59 / 61
#     4096 x 34592   936 / 794      2048 x 19360   182 / 130      1024 x 19360    81 / 75
APART_IN_OUTPUTS = 1 << 24
# The last product, by rows and by K (3072 + 14336, 1536 + 8192, 3072 + 3584 into 4096 or 2048 features), 256 /
# 512 / 2048 rows: 113 / 70, 176 / 100, 377 / 239; 28 / 43, 33 / 47, 78 / 87; 25 / 40, 41 / 45, 91 / 98.  (Up to
# 128 rows a long K goes to the engine's own product in pieces.)
APART_OUT_ROWS, APART_OUT_K = 128, 12288


def _aligned(count: int) -> int:
    return -(-count // ROW_STEP) * ROW_STEP


class JointProducts:
    """The two joint products of a mixer and a feed-forward (`partner`; None: the mixer alone)."""

    def __init__(self, mixer: Mixer, partner: FeedForward | None, dtype: torch.dtype) -> None:
        if not getattr(mixer, "can_join", False):
            raise ValueError(f"{type(mixer).__name__} does not say that its products can be made together with others")
        self.mixer, self.partner, self.dtype = mixer, partner, dtype
        self.hidden_size = mixer.joint_input.in_features
        self.ff = partner.gate_up.out_splits[0] if partner is not None else 0
        limit, slope = partner.joint_limits if partner is not None else (0.0, 1.0)
        self.layout = mixer.joint_layout(self.ff, limit, slope)
        self.mixer_columns = mixer.joint_input.padded_features
        self.inner = mixer.joint_output.in_features
        self.input_weight: torch.Tensor | None = None
        self.output_weight: torch.Tensor | None = None

    def join(self) -> None:
        """Stack the loaded weights and leave both parts views of them."""
        first, last = self.mixer.joint_input, self.mixer.joint_output
        blocks = [first.weight]
        if self.partner is not None:
            blocks.append(self.partner.gate_up.weight)
        rows = sum(block.shape[0] for block in blocks)
        stacked = first.weight.new_zeros((_aligned(rows), self.hidden_size))
        torch.cat(blocks, dim=0, out=stacked[:rows])
        first.weight = stacked[: self.mixer_columns]
        inner = self.inner + self.ff
        beside = last.weight.new_zeros((last.out_features, _aligned(inner)))
        beside[:, : self.inner] = last.weight
        last.weight = beside[:, : self.inner]
        if self.partner is not None:
            self.partner.gate_up.weight = stacked[self.mixer_columns: rows]
            beside[:, self.inner: inner] = self.partner.down.weight
            self.partner.down.weight = beside[:, self.inner: inner]
        self.input_weight, self.output_weight = stacked, beside[:, :inner]

    def wants_scaled_rows(self, rows: int) -> bool:
        """As `Mixer.wants_scaled_rows`: where the first product runs as the kernel that applies the rows' factors."""
        rotation = self.mixer.rotation()
        return (
            self.dtype == torch.bfloat16
            and rotation is not None
            and ops.layer_in_rows_fit(self.layout, *rotation)
            and ops.scaled_rows_product_takes(rows, self.input_weight, self.hidden_size)
        )

    def inner_rows(self, h, ctx: StepContext, cache: LayerCache, writes_cache: bool) -> torch.Tensor:
        """`[mix | act]` of the rows h, one row a token (rows may be strided): what the last product reads."""
        assert self.input_weight is not None, "joint products used before their weights were stacked"
        rows = h.values if isinstance(h, ops.ScaledRows) else h
        joined = torch.empty((rows.shape[0], _aligned(self.inner + self.ff)), dtype=self.dtype, device=rows.device)
        mixed, activated = joined[:, : self.inner], joined[:, self.inner: self.inner + self.ff]
        rotation = self.mixer.rotation()
        if rotation is not None and ops.layer_in_takes(h, self.input_weight, self.layout, *rotation):
            self.mixer.forward_layer_in(h, self.input_weight, self.layout, ctx, cache, writes_cache, activated, mixed)
        else:
            h = h.finish() if isinstance(h, ops.ScaledRows) else h
            if self.partner is not None and self.dtype == torch.bfloat16 and rows.shape[0] * self.input_weight.shape[0] >= APART_IN_OUTPUTS:
                own, gated = ops.linear(h, self.mixer.joint_input.weight), ops.linear(h, self.partner.gate_up.weight)
            else:
                columns = ops.linear(h, self.input_weight)
                own, gated = columns[:, : self.mixer_columns], columns[:, self.mixer_columns: self.mixer_columns + 2 * self.ff]
            self.mixer.forward_projected(own, ctx, cache, writes_cache, mixed)
            if self.partner is not None:
                self.partner.forward_projected(gated, activated)
        return joined[:, : self.inner + self.ff]

    def apart_out(self, rows: int) -> bool:
        """Whether the last product of so many rows is made in its two parts."""
        return (self.partner is not None and self.dtype == torch.bfloat16 and rows > APART_OUT_ROWS
                and self.inner + self.ff >= APART_OUT_K)

    def outputs(self, joined: torch.Tensor) -> tuple[torch.Tensor, torch.Tensor]:
        """The two parts of the last product of `inner_rows`."""
        assert self.partner is not None
        return (ops.linear(joined[:, : self.inner], self.mixer.joint_output.weight),
                ops.linear(joined[:, self.inner:], self.partner.down.weight))
