"""minGRU: a recurrence whose update gate and candidate do not look at its state.

    z = sigmoid(W_z h + b_z),   u = W_x h + b_x,   c = u + 1/2 where u >= 0 and sigmoid(u) where u < 0
    S <- (1 - z) S + z c                              (element by element, from zero)
    y = W_o (S * silu(W_g h))

Since no gate reads S, a step is an affine map of S that is known beforehand, and a prompt's maps are composed in
parallel.  A request's S lives in float32 in its state slot and is carried from step to step; gates, candidate, state and
the output's gate are float32 in both engines.
"""

from __future__ import annotations

import torch

from ..kernels import ops
from ..kernels.stages import stage
from ..weights.spec import MATRIX, VECTOR, Init, WeightSpec
from .base import Fetch, FixedStateSpec, LayerCache, Runtime
from .rows_mixer import RowsMixer


class MinGRU(RowsMixer):
    graph_safe = True
    input_label = "z/x/g"

    ROLES = {"z": "z", "x": "x", "g": "g", "o": "o", "z_bias": "z.b", "x_bias": "x.b"}

    def __init__(self, prefix: str, hidden_size: int, width: int, names: dict[str, str] | None = None,
                 suffix: str = "weight") -> None:
        """``names``: role -> the checkpoint's name under the prefix (the matrices' names are followed by ``suffix``
        unless it is empty; the biases are whole names)."""
        super().__init__(prefix)
        unknown = set(names or {}) - set(self.ROLES)
        if unknown:
            raise ValueError(f"{prefix}: unknown tensor roles {sorted(unknown)}; known: {sorted(self.ROLES)}")
        self.names = {**self.ROLES, **(names or {})}
        self.suffix = str(suffix)
        self.hidden_size, self.width = int(hidden_size), int(width)
        self.row_width, self.mixed_width = 3 * self.width, self.width

    def _matrix(self, role: str) -> str:
        return self.name(f"{self.names[role]}.{self.suffix}" if self.suffix else self.names[role])

    def weight_specs(self) -> list[WeightSpec]:
        specs = [WeightSpec(self._matrix(role), (self.width, self.hidden_size), MATRIX) for role in ("z", "x", "g")]
        specs += [WeightSpec(self.name(self.names["z_bias"]), (self.width,), VECTOR, Init(-1.0, 1.0)),
                  WeightSpec(self.name(self.names["x_bias"]), (self.width,), VECTOR, Init(0.0, 0.3)),
                  WeightSpec(self._matrix("o"), (self.hidden_size, self.width), MATRIX)]
        return specs

    def input_matrices(self, fetch: Fetch) -> list[torch.Tensor]:
        return [fetch(self._matrix(role)) for role in ("z", "x", "g")]

    def output_matrix(self, fetch: Fetch) -> torch.Tensor:
        return fetch(self._matrix("o"))

    def load_mixing(self, fetch: Fetch, runtime: Runtime) -> None:
        self.z_bias, self.x_bias = fetch(self.name(self.names["z_bias"])), fetch(self.name(self.names["x_bias"]))

    def cache_spec(self) -> FixedStateSpec:
        return FixedStateSpec((self.width,), torch.float32)

    def mix(self, rows: torch.Tensor, step, cache: LayerCache | None, out: torch.Tensor, scale: float) -> None:
        if cache is None or cache.state is None:
            raise ValueError(f"{self.prefix}: the recurrence needs a state slot per request")
        with stage("gated recurrence"):
            ops.min_gru(rows, self.z_bias, self.x_bias, step, cache.state, scale, out)
