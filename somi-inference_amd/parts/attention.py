"""Grouped-query attention over the paged cache.

Reference: somi_inference/models/qwen2.py:252-300 (q/k/v projections with bias,
o projection without, heads as contiguous head_dim blocks of the projection,
rotary encoding on q and k before k is cached), :158-186 (causal softmax
attention, scale head_dim^-0.5, query head h reads key/value head
h // (nq / nkv)) and somi_inference/core/paged_attention.py:352-413 (the same
over cache pages).  The reference has one function for whole prompts that never
reads the cache and one for single decoded tokens; here one kernel contract
serves any mix: keys and values of the step's tokens are written to their pages
first, then every token attends over its request's pages up to its own position.
"""

from __future__ import annotations

import torch

from ..kernels import attention as attention_kernels
from ..kernels import linear as linear_kernels
from ..kernels import ops
from ..kernels.stages import stage
from ..weights.spec import MATRIX, VECTOR, Init, WeightSpec
from .base import Fetch, LayerCache, Mixer, PagedKVSpec, PartSpec, PositionEncoding, Runtime
from .linear import NormedRows, Projection
from .registry import build_part


class GroupedQueryAttention(Mixer):
    graph_safe = True
    takes_normed_rows = True      # x only goes through the q/k/v projection, which norms rows while loading them
    entry_split = attention_kernels.DECODE_PORTION    # longer portions take the tile kernel, the rest the decode kernel

    def __init__(self, prefix: str, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int,
                 position: PartSpec, qkv_bias: bool = True, out_bias: bool = False,
                 window: int | None = None, scale: float | None = None, shares_cache: bool = False,
                 names: dict[str, str] | None = None, values: str = "projection", qk_norm: str | None = None,
                 norm_eps: float = 1e-6, suffix: str = "weight", value_dim: int | None = None, chunk: int | None = None,
                 softcap: float | None = None, sink: bool = False) -> None:
        """``names``: what the checkpoint calls this part's tensors, role -> name under the prefix.  Roles: ``q``,
        ``k``, ``v``, ``o`` (defaults ``q_proj`` ... ``o_proj``), ``position`` (``rotary_emb``), and ``qkv`` for a
        checkpoint that stores the three projections as one matrix, q rows first, then k, then v.

        ``values``: "projection" (a value projection of its own) or "keys" (there is none: a token's values are its
        keys as projected, before any norm).  ``qk_norm``: None, or "projection": q and k are each RMS-normed over the
        whole projection, all heads at once, with a weight of that size (roles ``q_norm``, ``k_norm``; ``norm_eps``
        inside the root); a rotation of the position encoding then comes after the norm.  ``suffix``: what follows a
        matrix's name in the checkpoint (empty: nothing; a bias is then ``<name>.bias`` all the same).

        ``value_dim``: channels of a value head, if they are not ``head_dim``.  ``chunk``: a query sees only the keys of its
        own run of that many positions.  ``softcap`` c: a scaled score s becomes c tanh(s / c).  ``sink``: a learned number a
        head (role ``sink``) whose exponential is part of the softmax's denominator."""
        super().__init__(prefix)
        if values not in ("projection", "keys") or qk_norm not in (None, "projection"):
            raise ValueError(f"{prefix}: values must be 'projection' or 'keys' and qk_norm None or 'projection', got "
                             f"{values!r} and {qk_norm!r}")
        self.values_are_keys, self.qk_norm, self.norm_eps = values == "keys", qk_norm, float(norm_eps)
        self.suffix = str(suffix)
        if (self.values_are_keys or qk_norm) and (shares_cache or qkv_bias or "qkv" in (names or {})):
            raise ValueError(f"{prefix}: values from the keys and a norm over the projections come without biases, "
                             f"a merged q/k/v matrix or a borrowed cache")
        self.value_dim = int(value_dim) if value_dim is not None else int(head_dim)
        self.chunk, self.softcap, self.has_sink = (int(chunk) if chunk else None), (float(softcap) if softcap else None), bool(sink)
        if self.softcap is not None and not self.softcap > 0.0:
            raise ValueError(f"{prefix}: a soft cap must be > 0, got {softcap}")
        if self.value_dim != int(head_dim) and (not qk_norm or self.values_are_keys):
            raise ValueError(f"{prefix}: value heads of another size than the keys' come with the norm over the projections and values of their own")
        unknown = set(names or {}) - set(self.ROLES) - {"qkv"}
        if unknown:
            raise ValueError(f"{prefix}: unknown tensor roles {sorted(unknown)}; known: {sorted(self.ROLES)} and 'qkv'")
        self.names = {**self.ROLES, **(names or {})}
        if num_heads % num_kv_heads != 0:
            # the reference's message (qwen2.py:116-123)
            raise ValueError(f"num_q_heads ({num_heads}) must be divisible by num_kv_heads ({num_kv_heads})")
        self.hidden_size, self.num_heads, self.num_kv_heads = int(hidden_size), int(num_heads), int(num_kv_heads)
        self.head_dim = int(head_dim)
        self.qkv_bias, self.out_bias = bool(qkv_bias), bool(out_bias)
        self.window = int(window) if window else None
        self.scale = float(scale) if scale is not None else self.head_dim ** -0.5
        self.shares_cache = bool(shares_cache)     # reads the cache another layer writes: no k/v of its own
        # what the pages keep: one size for keys and values, and, where a kernel of its own lays the heads out, one that the
        # matrix-core kernels take (a multiple of 16 from 32 on)
        self.kept_dim = self.head_dim
        if self.qk_norm and not self.values_are_keys:
            self.kept_dim = max(32, (max(self.head_dim, self.value_dim) + 15) // 16 * 16)
            if self.kept_dim > self.MAX_KEPT:
                raise ValueError(f"{prefix}: heads of {head_dim} and {self.value_dim} channels; at most {self.MAX_KEPT} are supported")
        self.score = ops.ScoreShape(self.softcap, self.chunk, None)
        self.position = build_part("position", position, prefix=self.name(self.names["position"]))
        if getattr(self.position, "pairing", "half") != "half":
            raise ValueError(f"{prefix}: this part's kernels rotate channel j with j + rotary_dim / 2 only")
        if getattr(self.position, "amplitude", 1.0) != 1.0:
            raise ValueError(f"{prefix}: this part's kernels take no amplitude on the rotation's cosines and sines")

    ROLES = {"q": "q_proj", "k": "k_proj", "v": "v_proj", "o": "o_proj", "position": "rotary_emb",
             "q_norm": "q_norm.weight", "k_norm": "k_norm.weight", "sink": "sink"}
    MAX_KEPT = 256              # the largest head size of the attention kernels

    def _weight(self, name: str) -> str:
        return self.name(f"{name}.{self.suffix}" if self.suffix else name)

    # ------------------------------------------------------------------ weights
    def _projections(self) -> list[tuple[str, int]]:
        """The checkpoint's input projections in the order their rows are stacked, with their widths."""
        q_width, kv_width = self.num_heads * self.head_dim, self.num_kv_heads * self.head_dim
        if self.shares_cache:
            return [(self.names["q"], q_width)]
        if "qkv" in self.names:
            return [(self.names["qkv"], q_width + 2 * kv_width)]
        if self.values_are_keys:
            return [(self.names["q"], q_width), (self.names["k"], kv_width)]
        return [(self.names["q"], q_width), (self.names["k"], kv_width), (self.names["v"], self.num_kv_heads * self.value_dim)]

    def weight_specs(self) -> list[WeightSpec]:
        specs = []
        for proj, width in self._projections():
            specs.append(WeightSpec(self._weight(proj), (width, self.hidden_size), MATRIX))
            if self.qkv_bias:
                specs.append(WeightSpec(self.name(f"{proj}.bias"), (width,), VECTOR))
        out = self.names["o"]
        specs.append(WeightSpec(self._weight(out), (self.hidden_size, self.num_heads * self.value_dim), MATRIX))
        if self.out_bias:
            specs.append(WeightSpec(self.name(f"{out}.bias"), (self.hidden_size,), VECTOR))
        if self.qk_norm:
            specs.append(WeightSpec(self.name(self.names["q_norm"]), (self.num_heads * self.head_dim,), VECTOR, Init(1.0, 0.1)))
            specs.append(WeightSpec(self.name(self.names["k_norm"]), (self.num_kv_heads * self.head_dim,), VECTOR, Init(1.0, 0.1)))
        if self.has_sink:
            specs.append(WeightSpec(self.name(self.names["sink"]), (self.num_heads,), VECTOR, Init(0.0, 1.0)))
        return specs + self.position.weight_specs()

    def load(self, fetch: Fetch, runtime: Runtime) -> None:
        super().load(fetch, runtime)
        names = [p for p, _ in self._projections()]
        self.qkv = Projection.stacked(
            [fetch(self._weight(p)) for p in names],
            [fetch(self.name(f"{p}.bias")) for p in names] if self.qkv_bias else None, label="q/k/v")
        out = self.names["o"]
        weight = fetch(self._weight(out))
        if self.kept_dim != self.value_dim and not self.values_are_keys and self.qk_norm:
            # the attention kernels' rows hold kept_dim channels a head, the ones past value_dim zero
            heads = weight.view(self.hidden_size, self.num_heads, self.value_dim)
            weight = torch.nn.functional.pad(heads, (0, self.kept_dim - self.value_dim)).reshape(self.hidden_size, -1).contiguous()
        self.out = Projection(weight,
                              fetch(self.name(f"{out}.bias")) if self.out_bias else None, label="o")
        if self.qk_norm:
            self.q_norm_weight = fetch(self.name(self.names["q_norm"]))
            self.k_norm_weight = fetch(self.name(self.names["k_norm"]))
        if self.has_sink:
            self.score = ops.ScoreShape(self.softcap, self.chunk, fetch(self.name(self.names["sink"])).contiguous())
        self.position.load(fetch, runtime)

    def flops(self, tokens: int, attended: int) -> float:
        """The projections, and q.k and p.v (two operations a product, head_dim channels, every query head) over the
        (token, key) pairs the step's tokens see."""
        return (self.qkv.flops(tokens) + self.out.flops(tokens)
                + 2.0 * self.num_heads * (self.head_dim + self.value_dim) * attended)

    # -------------------------------------------------------------------- cache
    def cache_spec(self) -> PagedKVSpec | None:
        if self.shares_cache:
            return None
        return PagedKVSpec(self.num_kv_heads, self.kept_dim, self.window, chunk=self.chunk)

    # ------------------------------------------------------------------ forward
    def forward(self, x: torch.Tensor, step, cache: LayerCache | None) -> torch.Tensor:
        if cache is None or cache.k is None:
            raise ValueError(f"{self.prefix}: attention needs a paged cache")
        view = step.paged[cache.group]
        nkv_new = 0 if self.shares_cache else self.num_kv_heads
        rotation = self.position.rotation_table()
        if self.qk_norm or self.values_are_keys:
            return self._forward_normed(x, step, view, cache, rotation)
        with stage(self.qkv.label):
            qkv = self._project_rotate_store(x, step, view, cache, rotation)     # a few rows: one kernel
        if qkv is None:
            qkv = self.qkv(x)                               # [N, (nq + 2 nkv) * D]
            with stage("position encoding, k/v into pages"):
                if rotation is None:
                    self.position.encode_qk(qkv, step, self.num_heads, nkv_new, self.head_dim)
                    inv_freq, rotary_dim = None, 0
                else:
                    inv_freq, rotary_dim = rotation
                ops.rope_kv_store(qkv, step.positions, view.slot_mapping if nkv_new else None, inv_freq, rotary_dim,
                                  self.num_heads, nkv_new, self.head_dim,
                                  cache.k if nkv_new else None, cache.v if nkv_new else None)
        with stage("attention"):
            attended = attention_kernels.paged_attention(
                qkv, self.num_heads, cache.k, cache.v, view.block_table, step,
                window=self.window or 0, scale=self.scale, score=self.score)
        return self.out.deferred(attended)        # the residual stream may add it in the kernel that computes it

    def _forward_normed(self, x, step, view, cache: LayerCache, rotation):
        """The path of a norm over the whole projections and of values that are the keys: the product, then one kernel
        that norms q (and turns it) and puts the normed keys and the values into their pages, then attention."""
        if type(self.position).encode_qk is not PositionEncoding.encode_qk:
            raise ValueError(f"{self.prefix}: only a rotation can follow a norm over the whole projection")
        if self.qk_norm and not self.values_are_keys:
            if hasattr(x, "materialize"):
                x = x.materialize()
            with stage(self.qkv.label):
                rows = linear_kernels.linear(x, self.qkv.weight, None, torch.float32)
            inv_freq, rotary_dim = rotation if rotation is not None else (None, 0)
            with stage("q/k norm, position encoding, k/v into pages"):
                q = ops.qk_norm_rope_store(rows, step.positions, view.slot_mapping, self.q_norm_weight, self.k_norm_weight,
                                           self.norm_eps, inv_freq, rotary_dim, self.num_heads, self.num_kv_heads,
                                           self.head_dim, self.value_dim, cache.k, cache.v)
            with stage("attention"):
                attended = attention_kernels.paged_attention(q, self.num_heads, cache.k, cache.v, view.block_table, step,
                                                             window=self.window or 0, scale=self.scale, score=self.score)
            return self.out.deferred(attended)
        if rotation is not None:
            raise ValueError(f"{self.prefix}: values that are the keys come without a rotation")
        rows = self.qkv(x)                              # [N, (nq + nkv) * D]
        with stage("q/k norm, k/v into pages"):
            if self.qk_norm:
                q_weight, k_weight, eps = self.q_norm_weight, self.k_norm_weight, self.norm_eps
            else:
                raise ValueError(f"{self.prefix}: values from the keys come with the norm over the projections")
            ops.qk_norm_store(rows, view.slot_mapping, q_weight, k_weight, eps, self.num_heads, self.num_kv_heads,
                              self.head_dim, self.values_are_keys, cache.k, cache.v)
        with stage("attention"):
            attended = attention_kernels.paged_attention(rows, self.num_heads, cache.k, cache.v, view.block_table, step,
                                                         window=self.window or 0, scale=self.scale, score=self.score)
        return self.out.deferred(attended)

    def _project_rotate_store(self, x, step, view, cache: LayerCache, rotation) -> torch.Tensor | None:
        """q of the step's tokens, rotated, with k and v in their pages, by the q/k/v product itself (up to 64 rows) or
        by the kernel that adds the sums of its K splits (some hundred rows); None where neither applies (many rows,
        float32, a head that is not rotated as a whole, no k/v of its own)."""
        if rotation is None or self.shares_cache:
            return None
        inv_freq, rotary_dim = rotation
        rows = x.shape[0]
        if (rotary_dim != self.head_dim or self.head_dim % 32 or cache.k.dtype != torch.bfloat16
                or not self.qkv.fusable(rows)):
            return None
        if isinstance(x, NormedRows):
            weighted, eps, stats = x.weighted, x.norm.eps, x.stats
        elif x.dtype == torch.bfloat16 and x.data_ptr() % 16 == 0:
            weighted, eps, stats = x, 0.0, None
        else:
            return None
        if rows > ops.FUSED_MAX_ROWS:
            # some hundred rows: the many-rows product shares a tile's K among workgroups, and the kernel that adds
            # their sums rotates and stores (more rows have tiles enough: the product, then the rotation)
            if ops.linear_big_splits(rows, self.qkv.out_features, self.qkv.in_features) <= 1:
                return None
            return ops.linear_big_rope_store(weighted, eps, stats, self.qkv.weight, self.qkv.bias, step.positions,
                                             view.slot_mapping, inv_freq, self.num_heads, self.num_kv_heads,
                                             self.head_dim, cache.k, cache.v)
        return ops.linear_rope_store(weighted, eps, stats, self.qkv.weight, self.qkv.bias, step.positions,
                                     view.slot_mapping, inv_freq, self.num_heads, self.num_kv_heads, self.head_dim,
                                     cache.k, cache.v)
