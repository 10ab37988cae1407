"""Mixture of experts: a router picks a few small feed-forwards per token; a shared one may run for all.

Router: ``z = W_r x`` in float32 and scores ``s = softmax(z)`` over all experts, or ``s = sigmoid(z)`` expert by expert
(``scores``).  The experts come in ``groups`` equal runs of neighbours; a run scores as its best expert, and only
experts of the ``keep`` best runs can be chosen.  Of those the ``top`` with the largest s are taken, weighted by s over
the sum of the chosen scores (+ 1e-20) or by s as it is (``normalize``; of a softmax over all experts that is the softmax
over the chosen ones).  With a ``correction`` tensor, one number an expert, the choice looks at s + correction and the
weights at s alone; with ``router_bias`` a stored number an expert is part of z.  A gated expert is

    g = min(W_gate x, limit);  u = clamp(W_up x, -limit, limit);  y = W_down (g sigmoid(alpha g) (u + shift))

without biases (no ``limit``, alpha 1 and shift 0: the plain ``silu(W_gate x) * (W_up x)``); one without a gate (``unit``
"squared_relu") is ``y = W_down relu(W_up x)^2``.  The output is the weighted
sum of the chosen experts' outputs or, with ``weight_on="input"``, the sum of the experts applied to ``w x`` (the
weight then scales the float32 sums of gate and up before the unit, which is not the same thing since the unit is not
linear); plus the shared expert's (the same form with sizes and a limit of its own), with ``shared_gate`` times sigmoid(w
x), one number a token.  The (token, expert) pairs are sorted by expert on the device, so that an
expert's rows are one block of the products' input; nothing of it is read by the host.
"""

from __future__ import annotations

import torch

from ..kernels import linear as linear_kernels
from ..kernels import ops
from ..kernels.stages import stage
from ..weights.spec import MATRIX, VECTOR, Init, WeightSpec
from .base import FeedForward, Fetch, Runtime
from .feed_forward import SwiGLU
from .linear import Projection


class ClampedGLU:
    """The constants of the experts' gated unit."""

    def __init__(self, limit: float | None, alpha: float = 1.702, shift: float = 1.0) -> None:
        self.limit = float(limit) if limit is not None else float("inf")       # no limit: nothing is clamped
        self.alpha, self.shift = float(alpha), float(shift)
        if not self.limit > 0.0:
            raise ValueError(f"a clamp limit must be > 0, got {limit}")
        self.plain = self.limit == float("inf") and self.alpha == 1.0 and self.shift == 0.0      # silu(g) u


class RoutedExperts(FeedForward):
    graph_safe = True

    ROLES = {"router": "router", "expert": "e", "shared": "shared", "gate": "gate", "up": "up", "down": "down",
             "correction": "correction", "bias": "router.b", "shared_gate": "sg"}

    UNITS = ("clamped_glu", "squared_relu")
    SCORES = ("softmax", "sigmoid")
    WEIGHT_ON = ("output", "input")

    def __init__(self, prefix: str, hidden_size: int, num_experts: int, top: int, expert_size: int, limit: float | None = None,
                 groups: int = 1, keep_groups: int = 1, shared_size: int | None = None, shared_limit: float | None = None,
                 alpha: float = 1.702, shift: float = 1.0, names: dict[str, str] | None = None, suffix: str = "weight",
                 scores: str = "softmax", normalize: bool = True, weight_on: str = "output", unit: str = "clamped_glu",
                 correction: bool = False, router_bias: bool = False, shared_gate: bool = False) -> None:
        """``names``: ``router``, the experts' stem (``e`` gives ``e0``, ``e1``, ...), ``shared``, the three matrices
        of an expert (two without a gate), ``correction``, ``bias`` and the shared expert's ``shared_gate``; ``suffix`` follows a matrix's name (empty: nothing)."""
        super().__init__(prefix)
        unknown = set(names or {}) - set(self.ROLES)
        if unknown:
            raise ValueError(f"{prefix}: unknown tensor roles {sorted(unknown)}; known: {sorted(self.ROLES)}")
        self.names = {**self.ROLES, **(names or {})}
        self.suffix = str(suffix)
        self.hidden_size, self.num_experts, self.top = int(hidden_size), int(num_experts), int(top)
        self.expert_size = int(expert_size)
        self.groups, self.keep_groups = int(groups), int(keep_groups)
        if self.groups < 1 or self.num_experts % self.groups or not 1 <= self.keep_groups <= self.groups:
            raise ValueError(f"{prefix}: {groups} groups (keep {keep_groups}) do not divide {num_experts} experts")
        if not 1 <= self.top <= self.keep_groups * (self.num_experts // self.groups):
            raise ValueError(f"{prefix}: top {top} does not fit the experts of {keep_groups} kept groups")
        if scores not in self.SCORES or weight_on not in self.WEIGHT_ON:
            raise ValueError(f"{prefix}: scores {scores!r} (one of {self.SCORES}), weight_on {weight_on!r} (one of {self.WEIGHT_ON})")
        self.scores, self.normalize, self.weight_on = scores, bool(normalize), weight_on
        if unit not in self.UNITS:
            raise ValueError(f"{prefix}: an expert's unit is one of {self.UNITS}, got {unit!r}")
        self.gated, self.has_correction = unit == "clamped_glu", bool(correction)
        self.has_bias, self.has_shared_gate = bool(router_bias), bool(shared_gate)
        if self.has_shared_gate and not shared_size:
            raise ValueError(f"{prefix}: a gate on the shared expert needs a shared expert")
        self.unit = ClampedGLU(limit, alpha, shift)
        self.shared_size = int(shared_size) if shared_size else None
        self.shared_unit = ClampedGLU(shared_limit if shared_limit is not None else limit, alpha, shift) if self.shared_size else None

    def _matrix(self, *parts: str) -> str:
        name = ".".join(parts)
        return self.name(f"{name}.{self.suffix}" if self.suffix else name)

    def _expert(self, index: int) -> str:
        return f"{self.names['expert']}{index}"

    def _ups(self) -> tuple[str, ...]:
        """The matrices in front of an expert's unit."""
        return ("gate", "up") if self.gated else ("up",)

    def weight_specs(self) -> list[WeightSpec]:
        h = self.hidden_size
        specs = [WeightSpec(self._matrix(self.names["router"]), (self.num_experts, h), VECTOR)]
        if self.has_correction:
            specs.append(WeightSpec(self.name(self.names["correction"]), (self.num_experts,), VECTOR, Init(0.0, 0.02)))
        if self.has_bias:
            specs.append(WeightSpec(self.name(self.names["bias"]), (self.num_experts,), VECTOR, Init(0.0, 0.1)))
        if self.has_shared_gate:
            specs.append(WeightSpec(self._matrix(self.names["shared"], self.names["shared_gate"]), (1, h), VECTOR))
        feeds = [(self._expert(e), self.expert_size) for e in range(self.num_experts)]
        if self.shared_size:
            feeds.append((self.names["shared"], self.shared_size))
        for feed, size in feeds:
            specs += [WeightSpec(self._matrix(feed, self.names[role]), (size, h), MATRIX) for role in self._ups()]
            specs.append(WeightSpec(self._matrix(feed, self.names["down"]), (h, size), MATRIX))
        return specs

    def load(self, fetch: Fetch, runtime: Runtime) -> None:
        super().load(fetch, runtime)
        self.router = fetch(self._matrix(self.names["router"]))            # float32: the router is computed in 32-bit
        if self.has_shared_gate:                                          # one row more of the router's product
            gate = fetch(self._matrix(self.names["shared"], self.names["shared_gate"]))
            self.router = torch.cat([self.router, gate], dim=0).contiguous()
        self.router_bias = fetch(self.name(self.names["bias"])) if self.has_bias else None
        self.correction = fetch(self.name(self.names["correction"])) if self.has_correction else None
        up, down = [], []
        for e in range(self.num_experts):
            up.append(torch.cat([fetch(self._matrix(self._expert(e), self.names[role])) for role in self._ups()], dim=0))
            down.append(fetch(self._matrix(self._expert(e), self.names["down"])))
        self.up = torch.stack(up).contiguous()                            # [experts, (2) F, H], gate rows first
        self.down = torch.stack(down).contiguous()                        # [experts, H, F]
        self.shared_up = self.shared_down = self.shared_glu = None
        if self.shared_size and self.gated and self.shared_unit.plain:
            # the plain gated unit: the product that ends in it
            self.shared_glu = SwiGLU(self.name(self.names["shared"]), self.hidden_size, self.shared_size,
                                     {role: self.names[role] for role in ("gate", "up", "down")}, suffix=self.suffix)
            self.shared_glu.load(fetch, runtime)
            self.shared_glu.gate_up.label, self.shared_glu.down.label = "shared gate_up", "shared down"
        elif self.shared_size:
            s = self.names["shared"]
            self.shared_up = Projection.stacked([fetch(self._matrix(s, self.names[role])) for role in self._ups()],
                                                label="shared gate_up" if self.gated else "shared up")
            self.shared_down = Projection(fetch(self._matrix(s, self.names["down"])), label="shared down")

    def flops(self, tokens: int, attended: int) -> float:
        matrices = len(self._ups()) + 1
        routed = 2.0 * matrices * tokens * self.top * self.expert_size * self.hidden_size
        shared = 2.0 * matrices * tokens * (self.shared_size or 0) * self.hidden_size
        return routed + shared + 2.0 * tokens * self.num_experts * self.hidden_size

    def forward(self, x, step=None) -> torch.Tensor:
        if hasattr(x, "materialize"):
            x = x.materialize()
        with stage("router"):
            gate = (torch.empty((x.shape[0],), dtype=torch.float32, device=x.device) if self.has_shared_gate else None)
            chosen, weight = ops.moe_route(x, self.router, self.top, self.groups, self.keep_groups, self.scores,
                                           self.normalize, self.correction, self.router_bias, gate)
            # bfloat16: the products run on the matrix cores, in tiles sized by the rows an expert gets in this step
            mfma = ops.moe_mfma_supported(x, self.up, self.down)
            rows = ops.moe_tile_rows(chosen.numel(), self.num_experts, mfma)
            order, _, tiles = ops.moe_align(chosen, self.num_experts, rows)
        input_weight = weight if self.weight_on == "input" else None
        with stage("experts gate_up" if self.gated else "experts up"):
            if self.gated:
                act = ops.moe_gate_up(x, self.up, tiles, order, self.top, self.unit.limit, self.unit.alpha, self.unit.shift,
                                      tile_rows=rows, mfma=mfma, input_weight=input_weight)
            else:
                act = ops.moe_up(x, self.up, tiles, order, self.top, tile_rows=rows, mfma=mfma, input_weight=input_weight)
        with stage("experts down"):
            pairs = ops.moe_down(act, self.down, tiles, order, weight if self.weight_on == "output" else None, self.top,
                                 tile_rows=rows, mfma=mfma)
        shared = self._shared(x) if self.shared_size else None
        with stage("experts' sum"):
            return ops.moe_combine(pairs, self.top, shared, gate)

    def _shared(self, x: torch.Tensor) -> torch.Tensor:
        if self.shared_glu is not None:
            y = self.shared_glu.forward(x)
            if hasattr(y, "projection"):
                with stage(y.projection.label):
                    return linear_kernels.linear(y.x, y.projection.weight, None, torch.float32)
            return y
        if not self.gated:
            up = self.shared_up(x, torch.float32)
            with stage("shared activation"):
                act = ops.squared_relu(up, self.runtime.dtype)
            return self.shared_down(act, torch.float32)
        gate_up = self.shared_up(x)
        with stage("shared activation"):
            gated = ops.clamped_glu(gate_up, self.shared_unit.limit, self.shared_unit.alpha, self.shared_unit.shift)
        return self.shared_down(gated)
