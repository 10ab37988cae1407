"""Plain Tomopel decoder: one slow function per mechanism, whole sequences at a time.

Written from the design's equations; it shares no code with the engine.  ``weights`` maps tensor names to
tensors of one floating type (float32, or float64 for a sharper yardstick), ``config`` is the parsed config.json.
Notation: ``x`` a stream ``[T, width]``, ``h`` a sublayer's input, ``i`` a query's position and ``j`` a key's.
"""

from __future__ import annotations

import math

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last dimension, eps inside the root."""
    return x / torch.sqrt(x.pow(2).mean(dim=-1, keepdim=True) + eps)


def norm_around_one(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """The root-mean-square norm whose stored weight is what is added to one."""
    return rms(x, eps) * (1.0 + w)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0.0)


# ------------------------------------------------------------------------------------- minGRU
def min_gru(h: torch.Tensor, weights: dict, prefix: str) -> torch.Tensor:
    """z and the candidate from the current token alone; S <- (1 - z) S + z c, element by element, from zero; the
    output is W_o (S silu(W_g h))."""
    z = torch.sigmoid(h @ weights[prefix + "z"].T + weights[prefix + "z.b"])
    u = h @ weights[prefix + "x"].T + weights[prefix + "x.b"]
    c = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    state = torch.zeros_like(z[0])
    states = []
    for t in range(h.shape[0]):
        state = (1.0 - z[t]) * state + z[t] * c[t]
        states.append(state)
    return (torch.stack(states) * silu(h @ weights[prefix + "g"].T)) @ weights[prefix + "o"].T


# ------------------------------------------------------------------------------------- attention with a distance bias
def bucket_of(n: int, buckets: int, farthest: int) -> int:
    """Distances below half the buckets have one each; the others share buckets whose edges grow geometrically up to
    ``farthest``.  Whole numbers only, so that a distance on an edge is on its own side of it: with h = buckets // 2
    and r = buckets - h, bucket h + s starts at the first n with (n / h)^r >= (farthest / h)^s."""
    half = buckets // 2
    if n < half:
        return n
    rest = buckets - half
    steps = 0
    while half + steps < buckets - 1 and n ** rest * half ** (steps + 1) >= farthest ** (steps + 1) * half ** rest:
        steps += 1
    return half + steps


def distance_bias(table: torch.Tensor, tokens: int, farthest: int) -> torch.Tensor:
    """[H, i, j] from ``table`` [B, H]: the row of the distance i - j (keys that are not seen get row 0)."""
    rows = torch.tensor([bucket_of(n, table.shape[0], farthest) for n in range(tokens)])
    i = torch.arange(tokens)
    n = (i[:, None] - i[None, :]).clamp(min=0)
    return table[rows[n]].permute(2, 0, 1)


def query_temperature(positions: torch.Tensor, coef: float, every: int) -> torch.Tensor:
    """1 + coef ln(floor((p + 1) / every) + 1)."""
    return 1.0 + coef * torch.log(torch.div(positions + 1, every, rounding_mode="floor").to(torch.float64) + 1.0)


def attention(h: torch.Tensor, weights: dict, prefix: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, D, Dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = rms((h @ weights[prefix + "q"].T).view(T, H, D), eps) * weights[prefix + "q.norm"]
    k = rms((h @ weights[prefix + "k"].T).view(T, G, D), eps) * weights[prefix + "k.norm"]
    v = rms((h @ weights[prefix + "v"].T).view(T, G, Dv), eps)
    if m.get("q_temp"):
        t = query_temperature(torch.arange(T), float(m["q_temp"]["coef"]), int(m["q_temp"]["every"]))
        q = q * t.to(q.dtype)[:, None, None]
    k = k.repeat_interleave(H // G, dim=1)
    v = v.repeat_interleave(H // G, dim=1)
    scores = torch.einsum("ihd,jhd->hij", q, k) * float(m["scale"])
    scores = scores + distance_bias(weights[prefix + "rel"], T, int(m["bias_max"]))
    i = torch.arange(T)
    scores = scores.masked_fill(i[None, :] > i[:, None], -math.inf)
    o = torch.einsum("hij,jhd->ihd", torch.softmax(scores, dim=-1), v)
    o = o * torch.sigmoid(h @ weights[prefix + "g"].T)[:, :, None]
    return o.reshape(T, H * Dv) @ weights[prefix + "o"].T


# ------------------------------------------------------------------------------------- Mamba-2
def causal_conv(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """Per channel over time; the last tap weighs the current token, zeros stand before the first."""
    T, width = x.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros(width - 1, x.shape[1], dtype=x.dtype), x])
    return sum(taps[:, j] * padded[j:j + T] for j in range(width)) + bias


def ssd(x: torch.Tensor, b: torch.Tensor, c: torch.Tensor, dt: torch.Tensor, a_log: torch.Tensor,
        d: torch.Tensor) -> torch.Tensor:
    """The recurrence: x [T, H, P], b and c [T, G, N], dt [T, H] (after the softplus) -> y [T, H, P]."""
    T, H, P = x.shape
    G, N = b.shape[1:]
    b, c = b.repeat_interleave(H // G, dim=1), c.repeat_interleave(H // G, dim=1)
    state = torch.zeros(H, N, P, dtype=x.dtype)
    rate = torch.exp(a_log)
    out = []
    for t in range(T):
        state = torch.exp(-rate * dt[t])[:, None, None] * state + dt[t][:, None, None] * b[t][:, :, None] * x[t][:, None, :]
        out.append((state * c[t][:, :, None]).sum(dim=1) + d[:, None] * x[t])
    return torch.stack(out)


def grouped_rms(y: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    """A row's ``groups`` equal parts, RMS-normed one by one."""
    T = y.shape[0]
    return rms(y.view(T, groups, -1), eps).reshape(T, -1)


def mamba2(h: torch.Tensor, weights: dict, prefix: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, P, N, G = int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"])
    inner = H * P
    z, xbc, dt = torch.split(h @ weights[prefix + "in"].T, [inner, inner + 2 * G * N, H], dim=1)
    xbc = silu(causal_conv(xbc, weights[prefix + "conv"], weights[prefix + "conv.b"]))
    x, b, c = torch.split(xbc, [inner, G * N, G * N], dim=1)
    dt = softplus(dt + weights[prefix + "dt_bias"])
    y = ssd(x.reshape(T, H, P), b.reshape(T, G, N), c.reshape(T, G, N), dt, weights[prefix + "A_log"], weights[prefix + "D"])
    y = grouped_rms(y.reshape(T, inner) * silu(z), int(m["norm_groups"]), eps) * weights[prefix + "norm"]
    return y @ weights[prefix + "o"].T


def parallel(h: torch.Tensor, weights: dict, prefix: str, m: dict, eps: float) -> torch.Tensor:
    return (float(m["left_scale"]) * attention(h, weights, prefix + "left.", m["left"], eps)
            + float(m["right_scale"]) * mamba2(h, weights, prefix + "right.", m["right"], eps))


# ------------------------------------------------------------------------------------- feed-forward
def dense(h: torch.Tensor, weights: dict, prefix: str) -> torch.Tensor:
    return (silu(h @ weights[prefix + "gate"].T) * (h @ weights[prefix + "up"].T)) @ weights[prefix + "down"].T


def expert(h: torch.Tensor, weights: dict, prefix: str) -> torch.Tensor:
    return torch.relu(h @ weights[prefix + "up"].T).pow(2) @ weights[prefix + "down"].T


def route(h: torch.Tensor, weights: dict, prefix: str, top: int) -> tuple[torch.Tensor, torch.Tensor, torch.Tensor]:
    """(chosen experts [T, top], their weights, how far the choice was from another one)."""
    scores = torch.softmax(h @ weights[prefix + "router"].T, dim=-1)
    choice = scores + weights[prefix + "correction"]
    ranked = choice.sort(dim=-1, descending=True)
    chosen = ranked.indices[:, :top]
    s = scores.gather(1, chosen)
    margin = (ranked.values[:, top - 1] - ranked.values[:, top] if top < choice.shape[1]
              else torch.full((h.shape[0],), math.inf, dtype=h.dtype))
    return chosen, s / (s.sum(dim=-1, keepdim=True) + 1e-20), margin


def experts(h: torch.Tensor, weights: dict, prefix: str, mlp: dict, margins: list | None = None) -> torch.Tensor:
    chosen, share, margin = route(h, weights, prefix, int(mlp["router"]["top"]))
    if margins is not None:
        margins.append(margin)
    rows = []
    for t in range(h.shape[0]):
        rows.append(sum(share[t, n] * expert(h[t], weights, f"{prefix}e{int(e)}.") for n, e in enumerate(chosen[t])))
    y = torch.stack(rows)
    return y + expert(h, weights, prefix + "shared.") if mlp.get("shared") else y


# ------------------------------------------------------------------------------------- the streams
def read_streams(streams: torch.Tensor, weights: dict, prefix: str) -> torch.Tensor:
    """u = sum_s in[s] x_s; streams: [S, T, width]."""
    return torch.einsum("s,stw->tw", weights[prefix + "in"], streams)


def write_streams(streams: torch.Tensor, y: torch.Tensor, weights: dict, prefix: str, mult: float) -> torch.Tensor:
    """x_t <- sum_s mix[s, t] x_s + mult out[t] y, every new stream from the old ones."""
    return (torch.einsum("st,sxw->txw", weights[prefix + "mix"], streams)
            + mult * weights[prefix + "out"][:, None, None] * y[None])


# ------------------------------------------------------------------------------------- the model
def forward(config: dict, weights: dict, tokens: list[int], dtype=torch.float64,
            margins: list | None = None) -> tuple[torch.Tensor, torch.Tensor]:
    """Logits [T, vocab] and the summed streams after every layer [layers, T, width].  ``margins`` collects, per routed
    layer, how far each token's choice of experts was from another one."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps, mult = float(config["norm"]["eps"]), float(config.get("residual_mult", 1.0))
    x = w["embed"][torch.tensor(tokens)] * float((config.get("embedding") or {}).get("scale", 1.0))
    hyper = "l0.hc1.in" in w
    streams = x[None].repeat(int(config.get("streams") or 1), 1, 1)
    after = []
    for n, layer in enumerate(config["layers"]):
        p, m = f"l{n}.", layer["mixer"]
        for sub in (1, 2):
            if sub == 2 and not layer.get("mlp"):
                continue
            u = read_streams(streams, w, f"{p}hc{sub}.") if hyper else streams[0]
            h = norm_around_one(u, w[f"{p}norm{sub}"], eps)
            if sub == 1:
                y = (parallel(h, w, p + "mix.", m, eps) if layer["type"] == "parallel" else min_gru(h, w, p + "mix."))
            elif layer["mlp"]["kind"] == "dense":
                y = dense(h, w, p + "mlp.")
            else:
                y = experts(h, w, p + "mlp.", layer["mlp"], margins)
            streams = write_streams(streams, y, w, f"{p}hc{sub}.", mult) if hyper else streams + mult * y[None]
        after.append(streams.sum(dim=0))
    x = norm_around_one(streams.sum(dim=0), w["final.norm"], eps)
    return x @ w["head"].T, torch.stack(after)


def load_folder(folder: str, dtype=torch.float32) -> tuple[dict, dict]:
    """(weights, config) of a model folder, floating tensors in ``dtype``."""
    import json
    import os

    from safetensors.torch import load_file
    with open(os.path.join(folder, "config.json"), "r", encoding="utf-8") as handle:
        config = json.load(handle)
    weights = {k: (v.to(dtype) if v.is_floating_point() else v)
               for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}
    return weights, config
