"""The residual stream of one step: float32 rows plus one pending, not yet added, delta.

The reference adds a sub-layer's output to the hidden state in the model dtype
(somi_inference/models/qwen2.py:333-339).  Here the sum is always float32, and
an add is deferred until the next norm so that one kernel does both
(``h += delta; x = norm(h)``).
"""

from __future__ import annotations

import torch

from ..kernels import ops
from ..kernels.stages import stage
from .base import Norm
from .linear import DeferredProduct, NormedRows


class ResidualStream:
    """For a few bfloat16 rows (decode steps) neither the add nor the norm is a kernel of its own: a part's
    last projection may arrive as a :class:`DeferredProduct`; ``normed(norm, lazy=True)`` then has it computed
    straight into ``h`` by a kernel that also leaves what the norm needs, and hands out :class:`NormedRows`,
    which the next projection scales while it multiplies."""

    def __init__(self, h: torch.Tensor) -> None:
        assert h.dtype == torch.float32 and h.dim() == 2
        self.h = h
        self._pending: torch.Tensor | DeferredProduct | None = None
        self._rounded: torch.Tensor | None = None   # h in the compute dtype, if whoever wrote h last left it
        self.lanes: torch.Tensor | None = None      # [S, N, H] float32 once a layer keeps several streams side by side

    def fan_out(self, count: int) -> torch.Tensor:
        """The stream as ``count`` streams side by side, ``[count, N, H]`` float32, all equal to ``h`` when they are
        made.  From then on the layers' arrangements update them in place, ``settle()`` gives their sum, and the
        single-stream calls (``add``, ``normed``) are refused."""
        if self.lanes is None:
            h = self.settle()
            self.lanes = ops.hc_step(h.unsqueeze(0), read=True, copies=count).view(count, *h.shape)
        if self.lanes.shape[0] != count:
            raise ValueError(f"the stream was fanned out into {self.lanes.shape[0]} streams, a layer asks for {count}")
        return self.lanes

    def _single(self) -> None:
        if self.lanes is not None:
            raise RuntimeError("the stream runs as several streams side by side; this layer's arrangement knows one")

    def rows(self, dtype: torch.dtype) -> torch.Tensor:
        """The stream itself in ``dtype``, for sublayers that read it without a norm (float32: the rows, not a copy)."""
        self._single()
        h = self.settle()
        if dtype == torch.float32:
            return h
        if self._rounded is None or self._rounded.dtype != dtype:
            self._rounded = h.to(dtype)
        return self._rounded

    def rewritten(self, rounded: torch.Tensor | None = None) -> None:
        """``h`` has been written in place; ``rounded``: the new rows in the compute dtype, if there are any."""
        self._rounded = rounded

    def add(self, delta: "torch.Tensor | DeferredProduct") -> None:
        """Queue ``h += delta``."""
        self._single()
        self.settle()
        self._rounded = None
        self._pending = delta

    def normed(self, norm: Norm, lazy: bool = False) -> "torch.Tensor | NormedRows":
        """norm(h) after any queued add.  ``lazy``: the caller's consumer takes :class:`NormedRows`."""
        self._single()
        if isinstance(self._pending, DeferredProduct):
            pending, self._pending = self._pending, None
            if lazy and getattr(norm, "fusable", False):
                return pending.add_to(self.h, norm)
            pending.add_to(self.h)
        with stage("residual add, norm"):
            if self._pending is not None:
                delta, self._pending = self._pending, None
                return norm.add_forward(self.h, delta)
            return norm.forward(self.h)

    def settle(self) -> torch.Tensor:
        """Apply a queued add and return the float32 rows (of several streams: their sum, the streams stay)."""
        if self.lanes is not None:
            with stage("residual add, norm"):
                return ops.hc_step(self.lanes, read=True)
        if isinstance(self._pending, DeferredProduct):
            self._pending.add_to(self.h)
        elif self._pending is not None:
            with stage("residual add, norm"):
                ops.residual_add(self.h, self._pending)
        self._pending = None
        return self.h
