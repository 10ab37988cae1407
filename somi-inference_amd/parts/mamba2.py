"""Mamba-2 (state-space duality): a recurrent mixer whose decay is one number a head and token.

One product of the input gives ``z | x | B | C | dt`` (inner = heads * value_dim channels of z and of x, ``groups *
state_dim`` of B and of C, one dt a head).  A short causal convolution with a bias and SiLU runs over the channels of x, B
and C (zeros stand before a request's first token, the last tap meets the token itself); then, head by head (head h reads
group ``h // (heads / groups)`` of B and C),

    dt  = softplus(dt + dt_bias)
    S   = exp(-exp(A_log) dt) S + dt B x^T;      y = S^T C + D x              (S: state_dim x value_dim, from zero)

y (the heads side by side) times ``silu(z)`` is cut into ``norm_groups`` equal parts, each part RMS-normed, the whole
times a weight, and projected by W_o.  A request's S and the ``taps - 1`` newest inputs of the convolution live in float32
in its state slot and are carried from step to step; the convolution, dt, the decay, the recurrence, the gate and the norm
are float32 in both engines.
"""

from __future__ import annotations

import torch

from ..kernels import ops
from ..kernels.stages import stage
from ..weights.spec import MATRIX, VECTOR, Init, WeightSpec
from .base import CompositeSpec, Fetch, FixedStateSpec, LayerCache, Runtime
from .rows_mixer import RowsMixer


class Mamba2(RowsMixer):
    graph_safe = True
    input_label = "z/x/B/C/dt"

    ROLES = {"in": "in", "o": "o", "conv": "conv", "conv_bias": "conv.b", "dt_bias": "dt_bias", "a_log": "A_log", "d": "D",
             "norm": "norm"}

    def __init__(self, prefix: str, hidden_size: int, num_heads: int, num_groups: int, state_dim: int, value_dim: int, taps: int,
                 norm_groups: int, eps: float, names: dict[str, str] | None = None, suffix: str = "weight") -> None:
        """``names``: role -> the checkpoint's name under the prefix (the two matrices' names are followed by ``suffix``
        unless it is empty; the others are whole names)."""
        super().__init__(prefix)
        unknown = set(names or {}) - set(self.ROLES)
        if unknown:
            raise ValueError(f"{prefix}: unknown tensor roles {sorted(unknown)}; known: {sorted(self.ROLES)}")
        self.names = {**self.ROLES, **(names or {})}
        self.suffix = str(suffix)
        self.hidden_size, self.num_heads, self.num_groups = int(hidden_size), int(num_heads), int(num_groups)
        self.state_dim, self.value_dim, self.taps = int(state_dim), int(value_dim), int(taps)
        self.norm_groups, self.eps = int(norm_groups), float(eps)
        self.inner = self.num_heads * self.value_dim
        if self.num_heads % self.num_groups or self.inner % self.norm_groups:
            raise ValueError(f"{prefix}: {num_groups} groups and {norm_groups} normed parts do not divide {num_heads} heads of {value_dim}")
        if not 1 <= self.taps <= ops.SHORT_CONV_MAX_TAPS:
            raise ValueError(f"{prefix}: a convolution of {taps} taps; 1 to {ops.SHORT_CONV_MAX_TAPS} are supported")
        self.channels = self.inner + 2 * self.num_groups * self.state_dim          # what passes the convolution
        self.row_width = self.inner + self.channels + self.num_heads
        self.mixed_width = self.inner

    # ------------------------------------------------------------------ weights
    def _matrix(self, role: str) -> str:
        return self.name(f"{self.names[role]}.{self.suffix}" if self.suffix else self.names[role])

    def weight_specs(self) -> list[WeightSpec]:
        def vector(role: str, shape: tuple, mean: float, std: float) -> WeightSpec:
            return WeightSpec(self.name(self.names[role]), shape, VECTOR, Init(mean, std))
        heads = (self.num_heads,)
        return [
            WeightSpec(self._matrix("in"), (self.row_width, self.hidden_size), MATRIX),
            vector("conv", (self.channels, self.taps), 0.3, 0.3), vector("conv_bias", (self.channels,), 0.0, 0.1),
            vector("dt_bias", heads, -2.0, 1.0), vector("a_log", heads, 0.0, 0.7), vector("d", heads, 1.0, 0.3),
            vector("norm", (self.inner,), 1.0, 0.1),
            WeightSpec(self._matrix("o"), (self.hidden_size, self.inner), MATRIX),
        ]

    def input_matrices(self, fetch: Fetch) -> list[torch.Tensor]:
        return [fetch(self._matrix("in"))]

    def output_matrix(self, fetch: Fetch) -> torch.Tensor:
        return fetch(self._matrix("o"))

    def load_mixing(self, fetch: Fetch, runtime: Runtime) -> None:
        def vector(role: str) -> torch.Tensor:
            return fetch(self.name(self.names[role])).contiguous()
        self.conv_taps, self.conv_bias = vector("conv"), vector("conv_bias")
        self.dt_bias, self.a_log, self.skip, self.norm_weight = vector("dt_bias"), vector("a_log"), vector("d"), vector("norm")

    def mixing_flops(self, tokens: int, attended: int) -> float:
        """The state's update and its product with C, two operations each on its state_dim x value_dim elements a head."""
        return 4.0 * self.inner * self.state_dim * tokens

    # -------------------------------------------------------------------- cache
    def cache_spec(self) -> CompositeSpec:
        """The state column by column (``[heads, value_dim, state_dim]``), and the convolution's kept inputs."""
        return CompositeSpec((
            ("state", FixedStateSpec((self.num_heads, self.value_dim, self.state_dim), torch.float32)),
            ("conv", FixedStateSpec((max(self.taps - 1, 1), self.channels), torch.float32)),
        ))

    # ------------------------------------------------------------------ forward
    def mix(self, rows: torch.Tensor, step, cache: LayerCache | None, out: torch.Tensor, scale: float) -> None:
        if cache is None or "state" not in cache.children or "conv" not in cache.children:
            raise ValueError(f"{self.prefix}: the recurrence needs a state slot per request")
        state, conv = cache.children["state"].state, cache.children["conv"].state
        z, xbc, dt = torch.split(rows, [self.inner, self.channels, self.num_heads], dim=1)
        with stage("convolution"):
            xbc = ops.conv_silu(xbc, self.conv_taps, self.conv_bias, conv, step)
        with stage("recurrence"):
            y = ops.ssd(xbc, dt, self.dt_bias, self.a_log, self.skip, step, state, self.num_groups)
        with stage("gate, norm"):
            ops.gated_group_norm(y, z, self.norm_weight, self.norm_groups, self.eps, scale, out)
