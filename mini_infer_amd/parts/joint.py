"""A layer whose sublayers read one norm, with their products made together.

Where a mixer and a gated feed-forward read the same rows h and their results are added up,

    y = W_o mix(W_m h) + W_down act(W_gate h, W_up h),

the two first products are one product with the stacked rows [W_m; W_gate; W_up], and, since
both results are sums, the two last ones are one product with the matrices side by side,

    y = [W_o | W_down] [mix(..); act(..)]

(the sum of the sublayers is then rounded once, not three times).  A layer is two products of
twice the size with the mixer's own work between them: at few rows the weights of a whole layer stream
through two launches, and the first of them ends with everything that follows it row by row
(`ops.layer_in`); a prompt's products are larger ones.

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
            columns = ops.linear(h, self.input_weight)
            self.mixer.forward_projected(columns[:, : self.mixer_columns], ctx, cache, writes_cache, mixed)
            if self.partner is not None:
                self.partner.forward_projected(columns[:, self.mixer_columns: self.mixer_columns + 2 * self.ff], activated)
        return joined[:, : self.inner + self.ff]
