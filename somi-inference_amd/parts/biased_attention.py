"""Grouped-query attention without a rotation: heads normed one by one, a learned bias by distance, a gate a head.

With H query heads over G key/value heads (query head h reads key/value head ``h // (H / G)``), ``dim`` query/key and
``value_dim`` value channels a head, and ``rms(u) = sqrt(mean(u^2) + eps)`` over a head's channels:

    q <- q / rms(q) * w_q * (1 + coef * ln(floor((p + 1) / every) + 1))      p: the query's position (``temperature``)
    k <- k / rms(k) * w_k;      v <- v / rms(v)
    s_h(i, j) = scale * q_h(i) . k(j) + rel[bucket(i - j), h]                j <= i
    o_h(i)    = sigmoid(g_h(i)) * sum_j softmax_j(s_h(i, j)) v(j),           then W_o on the concatenated heads

``bucket`` gives each distance below half of the table's rows a row of its own and spreads the others over the rest in
geometric steps up to ``bias_max``.  Norms, temperature, scores, softmax and gate are float32 in both engines; q and the
cached keys and values (as normed) take the engine's type.

The keys and values go through the engine's paged attention kernels, which take the bias as a table by distance
relative to what far keys get; those kernels have one head size, so heads whose key and value sizes differ (or do not fit
the matrix cores) are kept with zeros behind them.
"""

from __future__ import annotations

import torch

from ..kernels import attention as attention_kernels
from ..kernels import ops
from ..kernels.stages import stage
from ..weights.spec import ANY_SIZE, MATRIX, VECTOR, Init, WeightSpec
from .base import Fetch, LayerCache, PagedKVSpec, Runtime
from .rows_mixer import RowsMixer


def distance_buckets(buckets: int, farthest: int) -> list[int]:
    """The bucket of every distance from 0 up to the first that lies in the last bucket.

    With h = buckets // 2 and r = buckets - h, bucket h + s starts where ``h (farthest / h)^(s / r)`` does; compared in
    whole numbers (``(n / h)^r >= (farthest / h)^s``), so that a distance that falls on a start is in that bucket whatever
    a logarithm rounds to."""
    half = buckets // 2
    rest = buckets - half
    if half < 1 or farthest <= half:
        raise ValueError(f"{buckets} distance buckets up to {farthest}: at least two, and a farthest distance beyond half of them")
    out, bucket, n = [], 0, 0
    while True:
        if n < half:
            bucket = n
        else:
            bucket = max(bucket, half)
            while bucket < buckets - 1 and n ** rest * half ** (bucket + 1 - half) >= farthest ** (bucket + 1 - half) * half ** rest:
                bucket += 1
        out.append(bucket)
        if bucket == buckets - 1:
            return out
        n += 1


class BiasedAttention(RowsMixer):
    graph_safe = True
    entry_split = attention_kernels.DECODE_PORTION
    input_label = "q/k/v/gate"
    MAX_KEPT = 256              # the largest head size of the attention kernels

    ROLES = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm", "rel": "rel"}

    def __init__(self, prefix: str, hidden_size: int, num_heads: int, num_kv_heads: int, dim: int, value_dim: int,
                 scale: float, eps: float, bias_max: int | None = None, buckets: int | None = None, qk_norm: bool = True,
                 value_norm: bool = True, temperature: tuple[float, int] | None = None, gate: bool = True,
                 names: dict[str, str] | None = None, suffix: str = "weight") -> None:
        """``bias_max`` None: no distance bias; ``buckets`` None: as many as the checkpoint's table has rows.
        ``temperature``: (coef, every) or None.  ``names``: role -> the checkpoint's name under the prefix (a matrix's
        name is followed by ``suffix`` unless it is empty; the norms and the table are whole names)."""
        super().__init__(prefix)
        unknown = set(names or {}) - set(self.ROLES)
        if unknown:
            raise ValueError(f"{prefix}: unknown tensor roles {sorted(unknown)}; known: {sorted(self.ROLES)}")
        self.names = {**self.ROLES, **(names or {})}
        self.suffix = str(suffix)
        if num_heads % num_kv_heads != 0:
            raise ValueError(f"{prefix}: {num_heads} query heads are no multiple of {num_kv_heads} key/value heads")
        self.hidden_size, self.num_heads, self.num_kv_heads = int(hidden_size), int(num_heads), int(num_kv_heads)
        self.dim, self.value_dim, self.scale, self.eps = int(dim), int(value_dim), float(scale), float(eps)
        if not self.scale > 0.0:
            raise ValueError(f"{prefix}: the scale of the scores must be > 0, got {scale}")
        self.bias_max = int(bias_max) if bias_max is not None else None
        self.buckets = int(buckets) if buckets else None
        self.qk_norm, self.value_norm, self.gate = bool(qk_norm), bool(value_norm), bool(gate)
        self.temperature = (float(temperature[0]), int(temperature[1])) if temperature is not None else None
        # one size for keys and values, and one that the matrix-core kernels take (a multiple of 16 from 32 on)
        self.kept_dim = max(32, (max(self.dim, self.value_dim) + 15) // 16 * 16)
        if self.kept_dim > self.MAX_KEPT:
            raise ValueError(f"{prefix}: heads of {self.dim} and {self.value_dim} channels; at most {self.MAX_KEPT} are supported")
        self.row_width = self.num_heads * self.dim + self.num_kv_heads * (self.dim + self.value_dim) + (self.num_heads if self.gate else 0)
        self.mixed_width = self.num_heads * self.value_dim

    # ------------------------------------------------------------------ weights
    def _matrix(self, role: str) -> str:
        return self.name(f"{self.names[role]}.{self.suffix}" if self.suffix else self.names[role])

    def _inputs(self) -> list[tuple[str, int]]:
        rows = [("q", self.num_heads * self.dim), ("k", self.num_kv_heads * self.dim), ("v", self.num_kv_heads * self.value_dim)]
        return rows + [("g", self.num_heads)] if self.gate else rows

    def weight_specs(self) -> list[WeightSpec]:
        specs = [WeightSpec(self._matrix(role), (width, self.hidden_size), MATRIX) for role, width in self._inputs()]
        specs.append(WeightSpec(self._matrix("o"), (self.hidden_size, self.mixed_width), MATRIX))
        if self.qk_norm:
            specs += [WeightSpec(self.name(self.names[role]), (self.dim,), VECTOR, Init(1.0, 0.1)) for role in ("q_norm", "k_norm")]
        if self.bias_max is not None:
            specs.append(WeightSpec(self.name(self.names["rel"]), (self.buckets or ANY_SIZE, self.num_heads), VECTOR, Init(0.0, 1.0)))
        return specs

    def input_matrices(self, fetch: Fetch) -> list[torch.Tensor]:
        return [fetch(self._matrix(role)) for role, _ in self._inputs()]

    def output_matrix(self, fetch: Fetch) -> torch.Tensor:
        return fetch(self._matrix("o"))

    def load_mixing(self, fetch: Fetch, runtime: Runtime) -> None:
        self.q_weight = fetch(self.name(self.names["q_norm"])) if self.qk_norm else None
        self.k_weight = fetch(self.name(self.names["k_norm"])) if self.qk_norm else None
        self.bias = None
        if self.bias_max is not None:
            table = fetch(self.name(self.names["rel"]))                        # [buckets, heads]
            self.buckets = int(table.shape[0])
            rows = torch.tensor(distance_buckets(self.buckets, self.bias_max), device=table.device)
            # by head and distance, relative to the last bucket: a softmax does not see what every key gets
            self.bias = (table[rows] - table[-1:]).T.contiguous()

    def mixing_flops(self, tokens: int, attended: int) -> float:
        return 2.0 * self.num_heads * (self.dim + self.value_dim) * attended

    # -------------------------------------------------------------------- cache
    def cache_spec(self) -> PagedKVSpec:
        return PagedKVSpec(self.num_kv_heads, self.kept_dim)

    # ------------------------------------------------------------------ forward
    def mix(self, rows: torch.Tensor, step, cache: LayerCache | None, out: torch.Tensor, scale: float) -> None:
        if cache is None or cache.k is None:
            raise ValueError(f"{self.prefix}: attention needs a paged cache")
        view = step.paged[cache.group]
        with stage("head norms, k/v into pages"):
            q = ops.head_norm_store(rows, step.positions, view.slot_mapping, self.q_weight, self.k_weight, self.value_norm,
                                    self.eps, self.temperature, self.num_heads, self.num_kv_heads, self.dim, self.value_dim,
                                    cache.k, cache.v)
        with stage("attention"):
            attended = attention_kernels.paged_attention(q, self.num_heads, cache.k, cache.v, view.block_table, step,
                                                         window=0, scale=self.scale, bias=self.bias)
        with stage("head gate"):
            gate = rows[:, self.row_width - self.num_heads:self.row_width] if self.gate else None
            ops.head_gate(attended, gate, self.num_heads, self.value_dim, scale, out)
