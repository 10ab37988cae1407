"""Mixers that work between two products: one of their input, one that projects what they leave.

``RowsMixer`` keeps the two products apart from the mixing itself, so that an arrangement of several such mixers on one
input (:mod:`parallel_mixer`) can stack their input matrices into one product and lay their results side by side in
front of one output product.
"""

from __future__ import annotations

import torch

from ..kernels import linear as linear_kernels
from ..kernels.stages import stage
from .base import Fetch, LayerCache, Mixer, Runtime
from .linear import Projection


class RowsMixer(Mixer):
    """A subclass says how wide its input rows and its mixed rows are (``row_width``, ``mixed_width``), gives its two
    matrices and mixes."""

    row_width: int          # columns of the input product
    mixed_width: int        # columns in front of the output product
    input_label = "inputs"
    hidden_size: int

    def input_matrices(self, fetch: Fetch) -> list[torch.Tensor]:
        """The matrices whose stacked rows are the input product, ``row_width`` rows of ``hidden_size`` in all."""
        raise NotImplementedError

    def output_matrix(self, fetch: Fetch) -> torch.Tensor:
        """``[hidden_size, mixed_width]``."""
        raise NotImplementedError

    def load_mixing(self, fetch: Fetch, runtime: Runtime) -> None:
        """The tensors that are neither of the two products'."""

    def mix(self, rows: torch.Tensor, step, cache: LayerCache | None, out: torch.Tensor, scale: float) -> None:
        """rows: [N, row_width] float32 sums of the input product, possibly columns of wider rows -> ``scale`` times the
        mixed rows into ``out`` [N, mixed_width] in the compute dtype, likewise."""
        raise NotImplementedError

    def mixing_flops(self, tokens: int, attended: int) -> float:
        return 0.0

    def load(self, fetch: Fetch, runtime: Runtime) -> None:
        super().load(fetch, runtime)
        self.inputs = Projection.stacked(self.input_matrices(fetch), label=self.input_label)
        self.out = Projection(self.output_matrix(fetch), label="o")
        self.load_mixing(fetch, runtime)

    def flops(self, tokens: int, attended: int) -> float:
        return (2.0 * tokens * self.hidden_size * (self.row_width + self.mixed_width) + self.mixing_flops(tokens, attended))

    def forward(self, x, step, cache: LayerCache | None):
        if hasattr(x, "materialize"):
            x = x.materialize()
        with stage(self.inputs.label):
            rows = linear_kernels.linear(x, self.inputs.weight, None, torch.float32)
        mixed = torch.empty((rows.shape[0], self.mixed_width), dtype=self.runtime.dtype, device=rows.device)
        self.mix(rows, step, cache, mixed, 1.0)
        return self.out.deferred(mixed)
