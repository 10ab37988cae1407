"""mLSTM: a matrix memory with exponential gates, a normaliser and a running maximum that keeps both in range.

Per head, with q = W_q h key_dim^(-1/2), k = W_k h (key_dim channels), v = W_v h (value_dim) and two numbers a token,

    i   = cap tanh((W_i h + b_i) / cap),     f = log sigmoid(cap tanh((W_f h + b_f) / cap))      (log gates)
    m_t = max(f + m_(t-1), i)                                                                    (from 0)
    S   = exp(f + m_(t-1) - m_t) S + exp(i - m_t) k v^T,     n likewise with k alone             (from zero)
    o   = S^T q / (max(|n . q|, exp(-m_t)) + 1e-6)

each head's o is divided by its root mean square, the concatenated heads are multiplied by one weight and by sigmoid(W_g h),
and projected by W_o.  S and n are one state of value_dim + 1 columns; they and m live in float32 in the request's state
slots and are carried from step to step.  Gates, maxima, the recurrence, the norm and the output's gate are float32 in both
engines.
"""

from __future__ import annotations

import torch

from ..kernels import ops
from ..kernels.stages import stage
from ..weights.spec import MATRIX, VECTOR, Init, WeightSpec
from .base import CompositeSpec, Fetch, FixedStateSpec, LayerCache, Runtime
from .rows_mixer import RowsMixer


class MLSTM(RowsMixer):
    graph_safe = True
    input_label = "q/k/v/g/gates"

    ROLES = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "i": "i", "f": "f", "i_bias": "i.b", "f_bias": "f.b", "norm": "norm"}
    GRANULE = 8                 # the input rows are padded to a multiple of this many columns

    def __init__(self, prefix: str, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, gate_cap: float, eps: float,
                 names: dict[str, str] | None = None, suffix: str = "weight") -> None:
        """``names``: role -> the checkpoint's name under the prefix (the matrices' names are followed by ``suffix`` unless
        it is empty; the biases and the norm are whole names)."""
        super().__init__(prefix)
        unknown = set(names or {}) - set(self.ROLES)
        if unknown:
            raise ValueError(f"{prefix}: unknown tensor roles {sorted(unknown)}; known: {sorted(self.ROLES)}")
        self.names = {**self.ROLES, **(names or {})}
        self.suffix = str(suffix)
        self.hidden_size, self.num_heads = int(hidden_size), int(num_heads)
        self.key_dim, self.value_dim = int(key_dim), int(value_dim)
        self.gate_cap, self.eps = float(gate_cap), float(eps)
        if not self.gate_cap > 0.0:
            raise ValueError(f"{prefix}: the gates' cap must be > 0, got {gate_cap}")
        if self.key_dim > ops.SSD_MAX_ROWS:
            raise ValueError(f"{prefix}: keys of {key_dim} channels; at most {ops.SSD_MAX_ROWS} are supported")
        qk, vv = self.num_heads * self.key_dim, self.num_heads * self.value_dim
        self.splits = [qk, qk, vv, vv, self.num_heads, self.num_heads]
        self.row_width = (sum(self.splits) + self.GRANULE - 1) // self.GRANULE * self.GRANULE
        self.mixed_width = vv

    # ------------------------------------------------------------------ weights
    def _matrix(self, role: str) -> str:
        return self.name(f"{self.names[role]}.{self.suffix}" if self.suffix else self.names[role])

    INPUTS = ("q", "k", "v", "g", "i", "f")

    def weight_specs(self) -> list[WeightSpec]:
        heads = (self.num_heads,)
        return [WeightSpec(self._matrix(role), (rows, self.hidden_size), MATRIX) for role, rows in zip(self.INPUTS, self.splits)] + [
            WeightSpec(self.name(self.names["i_bias"]), heads, VECTOR, Init(-1.0, 1.0)),
            WeightSpec(self.name(self.names["f_bias"]), heads, VECTOR, Init(3.0, 1.0)),
            WeightSpec(self.name(self.names["norm"]), (self.mixed_width,), VECTOR, Init(1.0, 0.1)),
            WeightSpec(self._matrix("o"), (self.hidden_size, self.mixed_width), MATRIX),
        ]

    def input_matrices(self, fetch: Fetch) -> list[torch.Tensor]:
        matrices = [fetch(self._matrix(role)) for role in self.INPUTS]
        spare = self.row_width - sum(self.splits)
        return matrices + [torch.zeros_like(matrices[0][:1]).repeat(spare, 1)] if spare else matrices

    def output_matrix(self, fetch: Fetch) -> torch.Tensor:
        return fetch(self._matrix("o"))

    def load_mixing(self, fetch: Fetch, runtime: Runtime) -> None:
        def vector(role: str) -> torch.Tensor:
            return fetch(self.name(self.names[role])).contiguous()
        self.i_bias, self.f_bias, self.norm_weight = vector("i_bias"), vector("f_bias"), vector("norm")

    def mixing_flops(self, tokens: int, attended: int) -> float:
        """The state's update and its product with q, two operations each on its key_dim x (value_dim + 1) elements a head."""
        return 4.0 * self.num_heads * self.key_dim * (self.value_dim + 1) * tokens

    # -------------------------------------------------------------------- cache
    def cache_spec(self) -> CompositeSpec:
        """The memory column by column with the normaliser as the last one, and the running maxima."""
        return CompositeSpec((
            ("state", FixedStateSpec((self.num_heads, self.value_dim + 1, self.key_dim), torch.float32)),
            ("top", FixedStateSpec((self.num_heads,), torch.float32)),
        ))

    # ------------------------------------------------------------------ forward
    def mix(self, rows: torch.Tensor, step, cache: LayerCache | None, out: torch.Tensor, scale: float) -> None:
        if cache is None or "state" not in cache.children or "top" not in cache.children:
            raise ValueError(f"{self.prefix}: the recurrence needs a state slot per request")
        state, top = cache.children["state"].state, cache.children["top"].state
        q, k, v, g, i, f = torch.split(rows[:, :sum(self.splits)], self.splits, dim=1)
        with stage("gates"):
            keep, write, floor = ops.mlstm_gates(i, f, self.i_bias, self.f_bias, self.gate_cap, step, top)
        with stage("recurrence"):
            y, den = ops.ssd_memory(q, k, v, step, state, keep=keep, write=write, scale=self.key_dim ** -0.5)
        with stage("norm, gate"):
            ops.norm_sigmoid_gate(y, g, self.norm_weight, self.num_heads, self.eps, scale, out, den, floor)
