"""Lightning attention: linear attention whose decay is one fixed number a head.

With q = silu(W_q h), k = silu(W_k h) (``heads x key_dim``) and v = silu(W_v h) (``heads x value_dim``), per head

    S = decay S + k v^T,     o = S^T q                          (S: key_dim x value_dim, from zero)

the concatenated heads are RMS-normed together, multiplied by one weight and by sigmoid(W_g h), and projected by W_o.  S lives
in float32 in the request's state slot and is carried from step to step; the recurrence, the norm and the output's gate are
float32 in both engines.
"""

from __future__ import annotations

from typing import Sequence

import torch

from ..kernels import ops
from ..kernels.stages import stage
from ..weights.spec import MATRIX, VECTOR, Init, WeightSpec
from .base import Fetch, FixedStateSpec, LayerCache, Runtime
from .rows_mixer import RowsMixer


class LightningAttention(RowsMixer):
    graph_safe = True
    input_label = "q/k/v/g"

    ROLES = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "norm": "norm"}

    def __init__(self, prefix: str, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, decay: Sequence[float],
                 eps: float, names: dict[str, str] | None = None, suffix: str = "weight") -> None:
        """``names``: role -> the checkpoint's name under the prefix (the matrices' names are followed by ``suffix`` unless
        it is empty; the norm is a whole name)."""
        super().__init__(prefix)
        unknown = set(names or {}) - set(self.ROLES)
        if unknown:
            raise ValueError(f"{prefix}: unknown tensor roles {sorted(unknown)}; known: {sorted(self.ROLES)}")
        self.names = {**self.ROLES, **(names or {})}
        self.suffix = str(suffix)
        self.hidden_size, self.num_heads = int(hidden_size), int(num_heads)
        self.key_dim, self.value_dim, self.eps = int(key_dim), int(value_dim), float(eps)
        self.decay = [float(d) for d in decay]
        if len(self.decay) != self.num_heads:
            raise ValueError(f"{prefix}: {len(self.decay)} decays for {num_heads} heads")
        if self.key_dim > ops.SSD_MAX_ROWS:
            raise ValueError(f"{prefix}: keys of {key_dim} channels; at most {ops.SSD_MAX_ROWS} are supported")
        qk, vv = self.num_heads * self.key_dim, self.num_heads * self.value_dim
        self.splits = [qk, qk, vv, vv]
        self.row_width, self.mixed_width = 2 * qk + 2 * vv, vv

    # ------------------------------------------------------------------ weights
    def _matrix(self, role: str) -> str:
        return self.name(f"{self.names[role]}.{self.suffix}" if self.suffix else self.names[role])

    INPUTS = ("q", "k", "v", "g")

    def weight_specs(self) -> list[WeightSpec]:
        return [WeightSpec(self._matrix(role), (rows, self.hidden_size), MATRIX) for role, rows in zip(self.INPUTS, self.splits)] + [
            WeightSpec(self.name(self.names["norm"]), (self.mixed_width,), VECTOR, Init(1.0, 0.1)),
            WeightSpec(self._matrix("o"), (self.hidden_size, self.mixed_width), MATRIX),
        ]

    def input_matrices(self, fetch: Fetch) -> list[torch.Tensor]:
        return [fetch(self._matrix(role)) for role in self.INPUTS]

    def output_matrix(self, fetch: Fetch) -> torch.Tensor:
        return fetch(self._matrix("o"))

    def load_mixing(self, fetch: Fetch, runtime: Runtime) -> None:
        self.norm_weight = fetch(self.name(self.names["norm"])).contiguous()
        self.decays = torch.tensor(self.decay, dtype=torch.float32, device=runtime.device)

    def mixing_flops(self, tokens: int, attended: int) -> float:
        """The state's update and its product with q, two operations each on its key_dim x value_dim elements a head."""
        return 4.0 * self.num_heads * self.key_dim * self.value_dim * tokens

    # -------------------------------------------------------------------- cache
    def cache_spec(self) -> FixedStateSpec:
        """The state column by column."""
        return FixedStateSpec((self.num_heads, self.value_dim, self.key_dim), torch.float32)

    # ------------------------------------------------------------------ forward
    def mix(self, rows: torch.Tensor, step, cache: LayerCache | None, out: torch.Tensor, scale: float) -> None:
        if cache is None or cache.state is None:
            raise ValueError(f"{self.prefix}: the recurrence needs a state slot per request")
        q, k, v, g = torch.split(rows, self.splits, dim=1)
        with stage("input activation"):
            ops.silu_columns_(rows[:, :sum(self.splits[:3])])
        with stage("recurrence"):
            y, _ = ops.ssd_memory(q, k, v, step, cache.state, keep=self.decays)
        with stage("norm, gate"):
            ops.norm_sigmoid_gate(y, g, self.norm_weight, 1, self.eps, scale, out)
