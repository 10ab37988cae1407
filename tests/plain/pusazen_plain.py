"""Plain Pusazen decoder: one slow function per mechanism, whole sequences at a time.

Written from the design's equations; it shares no code with the engine.  ``weights`` maps tensor names to
tensors of one floating type (float32, or float64 for a sharper yardstick), ``config`` is the parsed config.json.
Notation: ``x`` the stream ``[T, width]``, which is also what a sublayer reads, ``i`` a query's position and ``j`` a key's.
"""

from __future__ import annotations

import math

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last dimension, eps inside the root."""
    return x / torch.sqrt(x.pow(2).mean(dim=-1, keepdim=True) + eps)


def norm_after(x: torch.Tensor, y: torch.Tensor, scale: torch.Tensor, alpha: float, w: torch.Tensor, eps: float) -> torch.Tensor:
    """norm(alpha x + scale y): a sublayer's scaled output joins the stream, and the sum is normed."""
    return rms(alpha * x + scale * y, eps) * w


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def log_sigmoid(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, max=0.0) - torch.log1p(torch.exp(-z.abs()))


# ------------------------------------------------------------------------------------- mLSTM
def mlstm_gates(x: torch.Tensor, weights: dict, prefix: str, cap: float) -> tuple[torch.Tensor, torch.Tensor]:
    """(log input gate, log forget gate), each [T, H]."""
    def capped(name: str) -> torch.Tensor:
        return cap * torch.tanh((x @ weights[prefix + name].T + weights[prefix + name + ".b"]) / cap)
    return capped("i"), log_sigmoid(capped("f"))


def mlstm_cell(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, i: torch.Tensor, f: torch.Tensor) -> torch.Tensor:
    """q, k [T, H, D], v [T, H, P], log gates [T, H] -> [T, H, P].  The matrix memory, the normaliser and the running
    maximum all start at zero."""
    T, H, D = q.shape
    memory = torch.zeros(H, D, v.shape[2], dtype=q.dtype)
    normaliser = torch.zeros(H, D, dtype=q.dtype)
    top = torch.zeros(H, dtype=q.dtype)
    out = []
    for t in range(T):
        before, top = top, torch.maximum(f[t] + top, i[t])
        keep, write = torch.exp(f[t] + before - top), torch.exp(i[t] - top)
        memory = keep[:, None, None] * memory + write[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        normaliser = keep[:, None] * normaliser + write[:, None] * k[t]
        read = (memory * q[t][:, :, None]).sum(dim=1)
        size = torch.maximum((normaliser * q[t]).sum(dim=1).abs(), torch.exp(-top)) + 1e-6
        out.append(read / size[:, None])
    return torch.stack(out)


def mlstm(x: torch.Tensor, weights: dict, prefix: str, m: dict, eps: float) -> torch.Tensor:
    T = x.shape[0]
    H, D, P = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = (x @ weights[prefix + "q"].T).view(T, H, D) * D ** -0.5
    k = (x @ weights[prefix + "k"].T).view(T, H, D)
    v = (x @ weights[prefix + "v"].T).view(T, H, P)
    o = mlstm_cell(q, k, v, *mlstm_gates(x, weights, prefix, float(m["gate_cap"])))
    o = rms(o, eps).reshape(T, H * P) * weights[prefix + "norm"]
    return (o * torch.sigmoid(x @ weights[prefix + "g"].T)) @ weights[prefix + "o"].T


# ------------------------------------------------------------------------------------- lightning attention
def lightning_cell(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: list[float]) -> torch.Tensor:
    """S <- decay_h S + k v^T, o = S^T q, from zero."""
    T, H, D = q.shape
    keep = torch.tensor([float(d) for d in decay], dtype=q.dtype)
    state = torch.zeros(H, D, v.shape[2], dtype=q.dtype)
    out = []
    for t in range(T):
        state = keep[:, None, None] * state + k[t][:, :, None] * v[t][:, None, :]
        out.append((state * q[t][:, :, None]).sum(dim=1))
    return torch.stack(out)


def lightning(x: torch.Tensor, weights: dict, prefix: str, m: dict, eps: float) -> torch.Tensor:
    T = x.shape[0]
    H, D, P = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = silu(x @ weights[prefix + "q"].T).view(T, H, D)
    k = silu(x @ weights[prefix + "k"].T).view(T, H, D)
    v = silu(x @ weights[prefix + "v"].T).view(T, H, P)
    o = lightning_cell(q, k, v, m["decay"]).reshape(T, H * P)
    o = rms(o, eps) * weights[prefix + "norm"] * torch.sigmoid(x @ weights[prefix + "g"].T)
    return o @ weights[prefix + "o"].T


# ------------------------------------------------------------------------------------- attention
def rotate(x: torch.Tensor, base: float, dims: int) -> torch.Tensor:
    """x [T, heads, D]: channel c < dims / 2 turns together with c + dims / 2 by the angle p base^(-2 c / dims)."""
    T, half = x.shape[0], dims // 2
    freq = torch.tensor([float(base) ** (-2.0 * c / dims) for c in range(half)], dtype=torch.float64)
    angle = (torch.arange(T, dtype=torch.float64)[:, None] * freq).to(x.dtype)[:, None, :]
    u, w, rest = x[..., :half], x[..., half:dims], x[..., dims:]
    return torch.cat([u * torch.cos(angle) - w * torch.sin(angle), w * torch.cos(angle) + u * torch.sin(angle), rest], dim=-1)


def chunk_mask(T: int, size: int) -> torch.Tensor:
    """True where query i sees key j: j <= i, and both in the same run of ``size`` positions counted from 0."""
    p = torch.arange(T)
    run = torch.div(p, size, rounding_mode="floor")
    return (p[None, :] <= p[:, None]) & (run[None, :] == run[:, None])


def sink_softmax(scores: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """Softmax over j of [H, i, j] whose denominator also holds exp(sink_h)."""
    top = torch.maximum(scores.amax(dim=-1, keepdim=True), sink[:, None, None])
    e = torch.exp(scores - top)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(sink[:, None, None] - top))


def attention(x: torch.Tensor, weights: dict, prefix: str, m: dict, eps: float) -> torch.Tensor:
    T = x.shape[0]
    H, G, D, P = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = rms(x @ weights[prefix + "q"].T, eps) * weights[prefix + "q.norm"]
    k = rms(x @ weights[prefix + "k"].T, eps) * weights[prefix + "k.norm"]
    v = (x @ weights[prefix + "v"].T).view(T, G, P).repeat_interleave(H // G, dim=1)
    base, dims = float(m["rot"]["base"]), int(m["rot"]["dims"])
    q = rotate(q.view(T, H, D), base, dims)
    k = rotate(k.view(T, G, D), base, dims).repeat_interleave(H // G, dim=1)
    scores = torch.einsum("ihd,jhd->hij", q, k) * float(m["scale"])
    cap = float(m["softcap"])
    scores = cap * torch.tanh(scores / cap)
    scores = scores.masked_fill(~chunk_mask(T, int(m["mask"]["size"])), -math.inf)
    o = torch.einsum("hij,jhd->ihd", sink_softmax(scores, weights[prefix + "sink"]), v)
    return o.reshape(T, H * P) @ weights[prefix + "o"].T


MIXERS = {"mlstm": mlstm, "lightning": lightning, "attention": attention}


# ------------------------------------------------------------------------------------- feed-forward
def dense(x: torch.Tensor, weights: dict, prefix: str) -> torch.Tensor:
    return torch.relu(x @ weights[prefix + "up"].T).pow(2) @ weights[prefix + "down"].T


def expert(x: torch.Tensor, weights: dict, prefix: str) -> torch.Tensor:
    return (silu(x @ weights[prefix + "gate"].T) * (x @ weights[prefix + "up"].T)) @ weights[prefix + "down"].T


def route(x: torch.Tensor, weights: dict, prefix: str, top: int) -> tuple[torch.Tensor, torch.Tensor, torch.Tensor]:
    """(chosen experts [T, top], their weights, how far the choice was from another one)."""
    z = x @ weights[prefix + "router"].T + weights[prefix + "router.b"]
    ranked = z.sort(dim=-1, descending=True)
    margin = (ranked.values[:, top - 1] - ranked.values[:, top] if top < z.shape[1]
              else torch.full((x.shape[0],), math.inf, dtype=x.dtype))
    return ranked.indices[:, :top], torch.softmax(ranked.values[:, :top], dim=-1), margin


def experts(x: torch.Tensor, weights: dict, prefix: str, mlp: dict, margins: list | None = None) -> torch.Tensor:
    chosen, share, margin = route(x, weights, prefix, int(mlp["router"]["top"]))
    if margins is not None:
        margins.append(margin)
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        y[t] = sum(share[t, n] * expert(x[t], weights, f"{prefix}e{int(e)}.") for n, e in enumerate(chosen[t]))
    if mlp.get("shared"):
        y = y + expert(x, weights, prefix + "shared.") * torch.sigmoid(x @ weights[prefix + "shared.sg"].T)
    return y


# ------------------------------------------------------------------------------------- the model
def forward(config: dict, weights: dict, tokens: list[int], dtype=torch.float64, margins: list | None = None,
            read_as: torch.dtype | None = None) -> tuple[torch.Tensor, torch.Tensor]:
    """Logits [T, vocab] and the stream after every layer [layers, T, width].  ``margins`` collects, per routed layer,
    how far each token's choice of experts was from another one.  ``read_as``: what the sublayers read is rounded to this
    type (how much rounding alone moves a row)."""
    def read(x: torch.Tensor) -> torch.Tensor:
        return x if read_as is None else x.to(read_as).to(dtype)

    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps, alpha = float(config["norm"]["eps"]), float(config["postln_alpha"])
    x = w["embed"][torch.tensor(tokens)]
    after = []
    for n, layer in enumerate(config["layers"]):
        p, mlp = f"l{n}.", layer.get("mlp")
        y = MIXERS[layer["type"]](read(x), w, p + "mix.", layer["mixer"], eps)
        x = norm_after(x, y, w[p + "ls1"], alpha, w[p + "norm1"], eps)
        if mlp:
            y = dense(read(x), w, p + "mlp.") if mlp["kind"] == "dense" else experts(read(x), w, p + "mlp.", mlp, margins)
            x = norm_after(x, y, w[p + "ls2"], alpha, w[p + "norm2"], eps)
        after.append(x)
    return read(rms(x, eps) * w["final.norm"]) @ w["head"].T * float(config["logit_scale"]), torch.stack(after)


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
