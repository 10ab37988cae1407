"""Two mixers side by side: both read the same input, and their outputs are joined.

``join`` "normed_mean": half the sum of the outputs, each first RMS-normed over the model width with a weight of its own.
``join`` "scaled_sum": ``left_scale * left + right_scale * right``.  Where both mixers work between two products
(:class:`RowsMixer`) the scaled sum needs no kernel of its own: their input matrices are stacked into one product, each
mixes its columns of the rows and leaves its result, scaled, in its columns of one row, and one product with the two
output matrices side by side projects and adds.

The two may be any registered mixers; what they keep per request is handed to the cache manager as one composite spec,
and each gets its own part of the layer's cache back.
"""

from __future__ import annotations

import math

import torch

from ..kernels import linear as linear_kernels
from ..kernels import ops
from ..kernels.stages import stage
from ..weights.spec import VECTOR, Init, WeightSpec
from .base import CompositeSpec, Fetch, LayerCache, Mixer, PartSpec, Runtime
from .linear import Projection
from .registry import build_part
from .rows_mixer import RowsMixer


class ParallelMixers(Mixer):
    """"normed_mean": y = (rms_norm(left(x)) * w_left + rms_norm(right(x)) * w_right) / 2, float32.  "scaled_sum": y =
    left_scale * left(x) + right_scale * right(x).  ``names``: the sub-prefixes of the two mixers (``left``, ``right``) and
    what follows them for the norms' weights (``out``)."""

    DEFAULT_NAMES = {"left": "left", "right": "right", "out": "out"}
    JOINS = ("normed_mean", "scaled_sum")

    def __init__(self, prefix: str, hidden_size: int, left: PartSpec, right: PartSpec, eps: float | None = None,
                 join: str = "normed_mean", left_scale: float = 1.0, right_scale: float = 1.0,
                 names: dict[str, str] | None = None) -> None:
        super().__init__(prefix)
        if join not in self.JOINS or (join == "normed_mean" and eps is None):
            raise ValueError(f"{prefix}: the outputs are joined by one of {self.JOINS} (the first needs 'eps'), got {join!r}")
        self.names = {**self.DEFAULT_NAMES, **(names or {})}
        self.hidden_size, self.join = int(hidden_size), join
        self.eps = float(eps) if eps is not None else 0.0
        self.scales = (float(left_scale), float(right_scale))
        self.left = build_part("mixer", left, prefix=self.name(self.names["left"]))
        self.right = build_part("mixer", right, prefix=self.name(self.names["right"]))
        self.stacked = join == "scaled_sum" and isinstance(self.left, RowsMixer) and isinstance(self.right, RowsMixer)
        self.graph_safe = bool(self.left.graph_safe and self.right.graph_safe)
        self.portion_granule = math.lcm(int(self.left.portion_granule), int(self.right.portion_granule))
        splits = {m.entry_split for m in (self.left, self.right) if m.entry_split is not None}
        if len(splits) > 1:
            raise ValueError(f"{prefix}: the two mixers cut a step's entries at different lengths {sorted(splits)}")
        self.entry_split = splits.pop() if splits else None

    def _out(self, side: str) -> str:
        return self.name(f"{self.names[side]}.{self.names['out']}")

    def weight_specs(self) -> list[WeightSpec]:
        specs = self.left.weight_specs() + self.right.weight_specs()
        if self.join == "normed_mean":
            specs += [WeightSpec(self._out(side), (self.hidden_size,), VECTOR, Init(1.0, 0.1)) for side in ("left", "right")]
        return specs

    def load(self, fetch: Fetch, runtime: Runtime) -> None:
        super().load(fetch, runtime)
        if self.stacked:
            for mixer in (self.left, self.right):
                mixer.runtime = runtime
                mixer.load_mixing(fetch, runtime)
            self.inputs = Projection.stacked(self.left.input_matrices(fetch) + self.right.input_matrices(fetch), label="inputs")
            self.out = Projection(torch.cat([self.left.output_matrix(fetch), self.right.output_matrix(fetch)], dim=1).contiguous(),
                                  label="o")
            return
        self.left.load(fetch, runtime)
        self.right.load(fetch, runtime)
        if self.join == "normed_mean":
            self.left_weight, self.right_weight = fetch(self._out("left")), fetch(self._out("right"))

    def flops(self, tokens: int, attended: int) -> float:
        return self.left.flops(tokens, attended) + self.right.flops(tokens, attended)

    def cache_spec(self) -> CompositeSpec | None:
        parts = tuple((side, spec) for side, spec in (("left", self.left.cache_spec()), ("right", self.right.cache_spec()))
                      if spec is not None)
        return CompositeSpec(parts) if parts else None

    def forward(self, x, step, cache: LayerCache | None):
        children = cache.children if cache is not None else {}
        if self.stacked:
            return self._forward_stacked(x, step, children)
        left = self.left.forward(x, step, children.get("left"))
        right = self.right.forward(x, step, children.get("right"))
        left, right = (y.materialize() if hasattr(y, "materialize") else y for y in (left, right))
        if self.join == "scaled_sum":
            with stage("scaled sum of the two mixers"):
                total = torch.zeros((left.shape[0], self.hidden_size), dtype=torch.float32, device=left.device)
                for y, scale in zip((left, right), self.scales):
                    ops.scaled_add(total, y if y.dtype == torch.float32 else y.to(torch.float32), None, scale)
                return total
        with stage("norms of the two mixers, mean"):
            return ops.normed_pair_mean(left, right, self.left_weight, self.right_weight, self.eps)

    def _forward_stacked(self, x, step, children):
        if hasattr(x, "materialize"):
            x = x.materialize()
        with stage(self.inputs.label):
            rows = linear_kernels.linear(x, self.inputs.weight, None, torch.float32)
        mixed = torch.empty((rows.shape[0], self.out.in_features), dtype=self.runtime.dtype, device=rows.device)
        row, at = 0, 0
        for mixer, side, scale in ((self.left, "left", self.scales[0]), (self.right, "right", self.scales[1])):
            mixer.mix(rows[:, row:row + mixer.row_width], step, children.get(side), mixed[:, at:at + mixer.mixed_width], scale)
            row, at = row + mixer.row_width, at + mixer.mixed_width
        return self.out.deferred(mixed)
