"""Decode and prefill throughput of the engine on one MI355X, at the layer sizes of Qwen2.5-7B by default.

``python bench.py --gpus 1 --steps K --warmup W`` builds a random-weights model in bfloat16, fills the cache of
``--batch`` requests by running their prompts through the engine's own generation loop (scheduler, step function,
sampler), then times exactly K of that loop's decode steps (one token per request per step) between two
synchronisations.  It prints ONE JSON line; ``value`` is decoded tokens per second.  The same line carries a
2,048-token prefill measurement, the decode step's HBM roofline figures, decode throughput at other numbers of
requests (``points``, with their step times, contexts and roofline fractions under ``point_details``) and, in the
default run, shorter measurements at the other configurations the headline is quoted beside (``extras``: the
14B sizes decoding and serving 32 requests with prompts in portions, the 32B sizes at 8,192 tokens, the 7B sizes at
32,768 tokens), each reported as an error instead of failing the line.

The model is whatever the registry builds from a config.json (``--config-json``, default: the ``--sizes`` of the
Qwen2.5 family): the bytes a decode step must read come from the tensors the model's parts declare and from its
cache specs, the operations of a prefill from the parts' own counts.  ``--stages`` adds the share of each named
stage (embedding, each product, attention, sampling) in eager steps.

The method follows the reference's benchmarks (warm-up, synchronise, wall clock, synchronise:
benchmarks/common.py:131-156; tokens/s = batch * iterations / time: benchmarks/bench_decode.py:241-247; the
engine run as a whole with its arrivals: benchmarks/bench_engine.py:181-283) with seeded random weights and seeded
uniform token ids in place of a downloaded checkpoint and a tokenizer-built workload.  The engine runs on one GPU;
for more it says so and exits with 2.
"""

from __future__ import annotations

import argparse
import gc
import json
import os
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, ROOT)

HBM_PEAK_GBS = 8000.0          # MI355X published HBM3E bandwidth
PEAK_FLOPS = {"bfloat16": 2.5e15, "float32": 157.3e12}   # dense MFMA peaks
POINT_BATCHES = (1, 64, 96, 128, 256)      # decode is also measured at these numbers of requests ("points")
POINT_MIN_STEPS = 16                       # a point is timed over at least this many steps


# layer sizes of the Qwen2.5 family: (layers, hidden, heads, kv heads, head_dim, intermediate, rms_norm_eps,
# vocabulary, tied LM head).  0.5b is the model the reference's own published figures are measured on.
LAYER_SIZES = {
    "0.5b": (24, 896, 14, 2, 64, 4864, 1e-6, 151936, True),
    "7b": (28, 3584, 28, 4, 128, 18944, 1e-6, 152064, False),
    "14b": (48, 5120, 40, 8, 128, 13824, 1e-5, 152064, False),
    "32b": (64, 5120, 40, 8, 128, 27648, 1e-6, 152064, False),
}
# layer sizes of Kamedra models that resemble real ones: (width, feed-forward, attention heads, key/value heads, size
# of one query/key map, value size, recurrent heads, their key size, their value size, rank of the decay's projection,
# window, kept first tokens, vocabulary).  Six layers: two recurrent ones, attention with a feed-forward, two recurrent
# ones, attention that borrows the first one's keys and values with a feed-forward.
KAMEDRA_SIZES = {
    "1b": (2048, 8192, 16, 4, 64, 128, 16, 64, 128, 64, 1024, 4, 32000),
    "7b": (4096, 14336, 32, 8, 64, 128, 32, 64, 128, 64, 2048, 4, 32000),
}


def kamedra_config_dict(sizes: str) -> dict:
    width, ff, heads, kv_heads, dim, vdim, r_heads, r_dim, r_vdim, rank, window, keep, vocab = KAMEDRA_SIZES[sizes]
    recurrent = {"type": "gla", "mlp": None, "mixer": {"heads": r_heads, "dim": r_dim, "vdim": r_vdim, "tau": 16.0, "rank": rank}}

    def attention(kv_from=None):
        mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "diff": 0.6, "scale": dim ** -0.5,
                 "mask": {"size": window, "keep_first": keep},
                 "rot": {"base": 500000.0, "dims": dim, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
        if kv_from is not None:
            mixer["kv_from"] = kv_from
        return {"type": "attention", "mixer": mixer, "mlp": {"kind": "dense", "ff": ff}}
    return {"architecture": "Kamedra", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "logit_softcap": 30.0,
            "layers": [recurrent, recurrent, attention(), recurrent, recurrent, attention(2)]}


def closest_config_dict(sizes: str) -> dict:
    """The Qwen2.5-style model of the same width, heads (one head of twice the map size for a head's two maps),
    key/value heads, feed-forward, vocabulary and number of layers."""
    width, ff, heads, kv_heads, dim, _, _, _, _, _, _, _, vocab = KAMEDRA_SIZES[sizes]
    return {"architectures": ["Qwen2ForCausalLM"], "model_type": "qwen2", "vocab_size": vocab, "hidden_size": width,
            "intermediate_size": ff, "num_hidden_layers": 6, "num_attention_heads": heads,
            "num_key_value_heads": kv_heads, "head_dim": 2 * dim, "rope_theta": 5e5, "rms_norm_eps": 1e-6,
            "tie_word_embeddings": True, "max_position_embeddings": 32768, "hidden_act": "silu", "attention_bias": False}


# layer sizes of Rusolorn models that resemble real ones: (width, attention heads, key/value heads, head size, window,
# recurrent value heads, recurrent q/k heads, their key size, their value size, taps, experts, experts a token, groups,
# kept groups, an expert's size, the shared expert's size, columns of the token input, vocabulary).  Six parallel layers.
RUSOLORN_SIZES = {
    "1b": (2048, 16, 4, 128, 1024, 16, 8, 128, 128, 4, 32, 4, 8, 4, 512, 1024, 128, 32000),
    "7b": (4096, 32, 8, 128, 2048, 32, 16, 128, 128, 4, 64, 6, 8, 4, 1024, 2048, 256, 32000),
}
RUSOLORN_LAYERS = 6


def rusolorn_config_dict(sizes: str) -> dict:
    (width, heads, kv_heads, dim, window, r_heads, r_groups, r_dim, r_vdim, taps, experts, top, groups, keep, ff, shared,
     side, vocab) = RUSOLORN_SIZES[sizes]
    layer = {"type": "parallel",
             "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5,
                                "mask": {"size": window}},
                       "right": {"heads": r_heads, "kv_heads": r_groups, "dim": r_dim, "vdim": r_vdim, "conv": taps}},
             "mlp": {"kind": "moe", "router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}},
                     "expert": {"ff": ff, "limit": 7.0}, "shared": {"ff": shared, "limit": 7.0}}}
    return {"architecture": "Rusolorn", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
            "residual_mult": 0.5, "token_side": {"dim": side}, "layers": [layer] * RUSOLORN_LAYERS}


def rusolorn_closest_config_dict(sizes: str) -> dict:
    """The closest model the engine had before: a Kamedra model of the same width, attention heads, window, recurrent
    heads and layers, whose layers take turns between the recurrent mixer and attention (a Rusolorn layer has both side
    by side) and whose dense feed-forward has the size of the experts a token uses plus the shared one."""
    (width, heads, kv_heads, dim, window, r_heads, _, r_dim, r_vdim, _, _, top, _, _, ff, shared, _, vocab) = RUSOLORN_SIZES[sizes]
    dense = {"kind": "dense", "ff": top * ff + shared}
    recurrent = {"type": "gla", "mlp": dense, "mixer": {"heads": r_heads, "dim": r_dim, "vdim": r_vdim, "tau": 16.0, "rank": 64}}
    attention = {"type": "attention", "mlp": dense,
                 "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim // 2, "vdim": dim, "diff": 0.6,
                           "scale": (dim // 2) ** -0.5, "mask": {"size": window, "keep_first": 0},
                           "rot": {"base": 500000.0, "dims": dim // 2}}}
    return {"architecture": "Kamedra", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "logit_softcap": 30.0,
            "layers": [recurrent, attention] * (RUSOLORN_LAYERS // 2)}


# layer sizes of Metitar models that resemble real ones: (width, attention heads, unrotated and rotated query/key
# channels a head, value size, latent size, query latent size, recurrent heads, their key size, their value size, taps,
# experts, experts a token, an expert's size, the shared expert's size, the dense feed-forward's size, columns of the
# token input, vocabulary).  Six layers: attention over the latent with a dense feed-forward, two recurrent layers with
# experts and a dense feed-forward, attention with experts, a recurrent layer with experts, attention that reads the
# fourth layer's latent with a dense feed-forward.
METITAR_SIZES = {
    "1b": (2048, 16, 128, 64, 128, 512, 768, 16, 128, 128, 4, 32, 4, 512, 1024, 4096, 128, 32000),
    "7b": (4096, 32, 128, 64, 128, 512, 1536, 32, 128, 128, 4, 64, 6, 1024, 2048, 8192, 256, 32000),
}
METITAR_LAYERS = 6


def metitar_config_dict(sizes: str) -> dict:
    (width, heads, dim, rot, vdim, rank, q_rank, r_heads, r_dim, r_vdim, taps, experts, top, ff, shared, dense_ff, side,
     vocab) = METITAR_SIZES[sizes]
    dense = {"kind": "dense", "ff": dense_ff}
    moe = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, "shared": {"ff": shared}}

    def attention(mlp, kv_from=None):
        mixer = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "q_rank": q_rank,
                 "scale": (dim + rot) ** -0.5,
                 "rot": {"base": 10000.0, "dims": rot, "scaling": {"factor": 40.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
        if kv_from is not None:
            mixer["kv_from"] = kv_from
        return {"type": "latent_attention", "mixer": mixer, "mlp": mlp}

    def recurrent(mlp):
        return {"type": "hgrn2", "mixer": {"heads": r_heads, "dim": r_dim, "vdim": r_vdim}, "mlp": mlp}
    return {"architecture": "Metitar", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0},
            "logit_scale": 1.0, "canon": {"taps": taps}, "token_side": {"dim": side},
            "layers": [attention(dense), recurrent(moe), recurrent(dense), attention(moe), recurrent(moe), attention(dense, 3)]}


def metitar_closest_config_dict(sizes: str) -> dict:
    """The closest model the engine had before: a Rusolorn model of the same width, attention heads and head size (a
    window longer than any context here, so its attention is causal over everything as well), recurrent heads and state
    size, experts, shared expert, token input and layers.  Each of its layers runs attention AND a recurrence and has
    experts; a Metitar layer has one mixer and experts in half of its layers."""
    (width, heads, dim, rot, vdim, rank, q_rank, r_heads, r_dim, r_vdim, taps, experts, top, ff, shared, dense_ff, side,
     vocab) = METITAR_SIZES[sizes]
    layer = {"type": "parallel",
             "mixer": {"left": {"heads": heads, "kv_heads": heads // 4, "dim": dim, "vdim": dim, "scale": dim ** -0.5,
                                "mask": {"size": 1 << 20}},
                       "right": {"heads": r_heads, "kv_heads": r_heads // 2, "dim": r_dim, "vdim": r_vdim, "conv": taps}},
             "mlp": {"kind": "moe", "router": {"experts": experts, "top": top, "groups": {"count": 1, "keep": 1}},
                     "expert": {"ff": ff, "limit": 7.0}, "shared": {"ff": shared, "limit": 7.0}}}
    return {"architecture": "Rusolorn", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
            "residual_mult": 0.5, "token_side": {"dim": side}, "layers": [layer] * METITAR_LAYERS}


# layer sizes of Gizilorn models that resemble real ones: (width, streams, attention heads, key/value heads, head size,
# the attention's window, latent-attention heads, unrotated and rotated query/key channels a head, value size, latent
# size, the latent attention's window, the dense feed-forward's size, vocabulary).  Six layers: latent attention, latent
# attention that reads the first layer's latent, two attention layers with mixed heads, latent attention, attention.
GIZILORN_SIZES = {
    "1b": (2048, 4, 16, 4, 128, 1024, 16, 128, 64, 128, 512, 4096, 4096, 32000),
    "7b": (4096, 4, 32, 8, 128, 2048, 32, 128, 64, 128, 512, 4096, 8192, 32000),
}
GIZILORN_LAYERS = 6


def gizilorn_config_dict(sizes: str) -> dict:
    (width, streams, heads, kv_heads, dim, window, l_heads, l_dim, rot, vdim, rank, l_window, ff, vocab) = GIZILORN_SIZES[sizes]
    dense = {"kind": "dense", "ff": ff}

    def latent(kv_from=None):
        mixer = {"heads": l_heads, "dim": l_dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": (l_dim + rot) ** -0.5,
                 "mask": {"size": l_window}, "rot": {"base": 100000.0, "dims": rot}}
        if kv_from is not None:
            mixer["kv_from"] = kv_from
        return {"type": "latent_attention", "mixer": mixer, "mlp": dense}
    attention = {"type": "attention", "mlp": dense,
                 "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "softcap": 30.0,
                           "mask": {"size": window}, "rot": {"base": 10000.0, "dims": dim}}}
    return {"architecture": "Gizilorn", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "streams": streams,
            "layers": [latent(), latent(0), attention, attention, latent(), attention]}


def gizilorn_closest_config_dict(sizes: str) -> dict:
    """The closest model the engine had before, for the latent attention, the dense feed-forwards and what stands
    between the sublayers: a Metitar model of six latent-attention layers of the same width, heads, head sizes and
    latent (with a query latent of three quarters of the width's half, a sink, and no window: it is causal over
    everything) and dense feed-forwards of the same size; no input convolution, no token input."""
    (width, streams, heads, kv_heads, dim, window, l_heads, l_dim, rot, vdim, rank, l_window, ff, vocab) = GIZILORN_SIZES[sizes]

    def latent(kv_from=None):
        mixer = {"heads": l_heads, "dim": l_dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "q_rank": 3 * width // 8,
                 "scale": (l_dim + rot) ** -0.5, "rot": {"base": 10000.0, "dims": rot}}
        if kv_from is not None:
            mixer["kv_from"] = kv_from
        return {"type": "latent_attention", "mixer": mixer, "mlp": {"kind": "dense", "ff": ff}}
    return {"architecture": "Metitar", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0},
            "logit_scale": 1.0, "layers": [latent(), latent(0), latent(), latent(), latent(), latent(4)]}


def gizilorn_closest_attention_config_dict(sizes: str) -> dict:
    """The closest model for the attention with mixed heads: a Qwen2.5-style model of the same width, heads, key/value
    heads, head size and window in every layer."""
    (width, streams, heads, kv_heads, dim, window, l_heads, l_dim, rot, vdim, rank, l_window, ff, vocab) = GIZILORN_SIZES[sizes]
    return {"architectures": ["Qwen2ForCausalLM"], "model_type": "qwen2", "vocab_size": vocab, "hidden_size": width,
            "intermediate_size": ff, "num_hidden_layers": GIZILORN_LAYERS, "num_attention_heads": heads,
            "num_key_value_heads": kv_heads, "head_dim": dim, "rope_theta": 1e4, "rms_norm_eps": 1e-6,
            "tie_word_embeddings": False, "max_position_embeddings": 32768, "hidden_act": "silu", "attention_bias": True,
            "use_sliding_window": True, "sliding_window": window, "max_window_layers": 0}


# layer sizes of Tomopel models that resemble real ones: (width, residual streams, attention heads, key/value heads, head
# size, recurrent heads, their value size, their state, groups of B and C, taps, minGRU width, experts, experts a token, an
# expert's size, the shared expert's size, the dense feed-forward's size, vocabulary).  Six layers: attention beside
# Mamba-2 in all but the fourth, which is a minGRU; a dense feed-forward in the first, routed experts in the others.
TOMOPEL_SIZES = {
    "1b": (2048, 2, 16, 4, 128, 32, 64, 128, 1, 4, 2048, 32, 4, 512, 1024, 4096, 32000),
    "7b": (4096, 2, 32, 8, 128, 64, 64, 128, 1, 4, 4096, 64, 6, 1024, 2048, 8192, 32000),
}
TOMOPEL_LAYERS, TOMOPEL_PARALLEL = 6, 5


def tomopel_config_dict(sizes: str) -> dict:
    (width, streams, heads, kv_heads, dim, r_heads, r_vdim, state, groups, taps, gru, experts, top, ff, shared, dense_ff,
     vocab) = TOMOPEL_SIZES[sizes]
    moe = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, "shared": {"ff": shared}}

    def parallel(mlp):
        return {"type": "parallel", "mlp": mlp, "mixer": {
            "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "bias_max": 128,
                     "buckets": 32, "q_temp": {"coef": 0.1, "every": 8192}},
            "right": {"heads": r_heads, "vdim": r_vdim, "state": state, "groups": groups, "conv": taps, "norm_groups": 1},
            "left_scale": 0.5, "right_scale": 0.5}}
    return {"architecture": "Tomopel", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
            "residual_mult": 0.5, "streams": streams,
            "layers": [parallel({"kind": "dense", "ff": dense_ff}), parallel(moe), parallel(moe),
                       {"type": "mingru", "mixer": {"width": gru}, "mlp": moe}, parallel(moe), parallel(moe)]}


def tomopel_closest_config_dict(sizes: str) -> dict:
    """The closest model the engine had before: a Rusolorn model of the same width, attention heads (its window holds every
    context measured here), recurrent state (as many elements a token and layer, in 128 x 128 heads), experts and layers;
    no token input."""
    (width, streams, heads, kv_heads, dim, r_heads, r_vdim, state, groups, taps, gru, experts, top, ff, shared, dense_ff,
     vocab) = TOMOPEL_SIZES[sizes]
    delta_heads = r_heads * r_vdim * state // (128 * 128)
    layer = {"type": "parallel",
             "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5,
                                "mask": {"size": 65536}},
                       "right": {"heads": delta_heads, "kv_heads": delta_heads // 2, "dim": 128, "vdim": 128, "conv": taps}},
             "mlp": {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": 7.0},
                     "shared": {"ff": shared, "limit": 7.0}}}
    return {"architecture": "Rusolorn", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
            "residual_mult": 0.5, "layers": [layer] * TOMOPEL_LAYERS}


def tomopel_closest_streams_config_dict(sizes: str) -> dict:
    """The closest model for what stands between the sublayers and for the dense feed-forward: a Gizilorn model of the
    same width and number of streams, with attention with mixed heads and dense feed-forwards of the same size."""
    (width, streams, heads, kv_heads, dim, r_heads, r_vdim, state, groups, taps, gru, experts, top, ff, shared, dense_ff,
     vocab) = TOMOPEL_SIZES[sizes]
    layer = {"type": "attention", "mlp": {"kind": "dense", "ff": dense_ff},
             "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5,
                       "mask": {"size": 512}, "rot": {"base": 10000.0, "dims": dim}}}
    return {"architecture": "Gizilorn", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "streams": streams,
            "layers": [layer] * TOMOPEL_LAYERS}


# layer sizes of Pusazen models that resemble real ones: (width, mLSTM heads, their key and value sizes, lightning heads, their
# key and value sizes, attention heads, key/value heads, head size, chunk, experts, experts a token, an expert's size, the
# shared expert's size, the dense feed-forward's size, vocabulary).  Six layers: three mLSTM, two attention, one lightning; a
# dense feed-forward in the first, routed experts in the others.  The states hold as many elements as the Mamba-2 states of the
# Tomopel model of the same name.
PUSAZEN_SIZES = {
    "1b": (2048, 8, 128, 256, 16, 128, 128, 16, 4, 128, 8192, 32, 4, 512, 1024, 8192, 32000),
    "7b": (4096, 16, 128, 256, 32, 128, 128, 32, 8, 128, 8192, 64, 6, 1024, 2048, 16384, 32000),
}
PUSAZEN_LAYERS = {"mlstm": 3, "attention": 2, "lightning": 1}


def pusazen_config_dict(sizes: str) -> dict:
    (width, m_heads, m_dim, m_vdim, l_heads, l_dim, l_vdim, heads, kv_heads, dim, chunk, experts, top, ff, shared, dense_ff,
     vocab) = PUSAZEN_SIZES[sizes]
    moe = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, "shared": {"ff": shared}}
    mixers = {"mlstm": {"heads": m_heads, "dim": m_dim, "vdim": m_vdim, "gate_cap": 15.0},
              "lightning": {"heads": l_heads, "dim": l_dim, "vdim": l_vdim, "decay": [1.0 - 2.0 ** -(2 + h % 8) for h in range(l_heads)]},
              "attention": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "softcap": 50.0,
                            "rot": {"base": 10000.0, "dims": dim // 2}, "mask": {"size": chunk}}}
    order = ("mlstm", "attention", "mlstm", "lightning", "mlstm", "attention")
    return {"architecture": "Pusazen", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "postln_alpha": 2.0, "logit_scale": 1.0,
            "layers": [{"type": kind, "mixer": mixers[kind], "mlp": moe if index else {"kind": "dense", "ff": dense_ff}}
                       for index, kind in enumerate(order)]}


def pusazen_closest_dense_config_dict(sizes: str) -> dict:
    """The closest model for the ungated dense feed-forward and for the norm behind a sublayer: a Metitar model of the same
    width whose layers all have a dense feed-forward of the same size."""
    (width, m_heads, m_dim, m_vdim, l_heads, l_dim, l_vdim, heads, kv_heads, dim, chunk, experts, top, ff, shared, dense_ff,
     vocab) = PUSAZEN_SIZES[sizes]
    layer = {"type": "hgrn2", "mixer": {"heads": l_heads, "dim": l_dim, "vdim": l_vdim}, "mlp": {"kind": "dense", "ff": dense_ff}}
    return {"architecture": "Metitar", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
            "layers": [layer] * 6}


# keys of a config.json that name sizes, in the order they are reported under "config" (flat, at most 20 keys)
SIZE_KEYS = ("hidden_size", "intermediate_size", "num_attention_heads", "num_key_value_heads", "head_dim",
             "vocab_size", "tie_word_embeddings")


def parse_args() -> argparse.Namespace:
    p = argparse.ArgumentParser(description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    p.add_argument("--gpus", type=int, default=1)
    p.add_argument("--steps", type=int, default=64)
    p.add_argument("--warmup", type=int, default=8)
    p.add_argument("--batch", type=int, default=8)
    p.add_argument("--context", type=int, default=4096, help="context length the timed decode steps end at")
    p.add_argument("--sizes", default="7b", choices=sorted(LAYER_SIZES),
                   help="layer sizes: Qwen2.5-7B (the default and the headline), -14B, -32B, or -0.5B (the model of the "
                        "reference's own published figures)")
    p.add_argument("--config-json", type=str, default=None,
                   help="a config.json of any registered architecture instead of --sizes")
    p.add_argument("--layers", type=int, default=None, help="run fewer layers than the configuration has")
    p.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    p.add_argument("--block-size", type=int, default=16)
    p.add_argument("--prefill-tokens", type=int, default=2048)
    p.add_argument("--seed", type=int, default=0)
    p.add_argument("--no-points", action="store_true", help="skip the decode points at other batch sizes (1, 64, 96, 128, 256)")
    p.add_argument("--no-prefill", action="store_true", help="skip the prefill measurement")
    p.add_argument("--no-peaks", action="store_true", help="skip the measurement of the machine's own peaks")
    p.add_argument("--no-extras", action="store_true",
                   help="skip the short measurements at the 14B and 32B sizes and at 32,768 tokens that the default run adds")
    p.add_argument("--extras-budget", type=float, default=300.0, metavar="SECONDS",
                   help="no further extra measurement is started once the run has taken this long")
    p.add_argument("--stages", action="store_true",
                   help="also time the named stages of an eager prefill and an eager decode step and report their shares")
    p.add_argument("--output-file", type=str, default=None, help="Append the result line to a JSONL file.")
    p.add_argument("--kamedra", default=None, choices=sorted(KAMEDRA_SIZES), metavar="SIZES",
                   help="instead of the default workload: prefill and decode of a Kamedra model (differential attention "
                        "with a window, gated linear attention) at these layer sizes, beside the Qwen2.5-style model of "
                        "equal width, heads, feed-forward and layers, each with its stage times")
    p.add_argument("--rusolorn", default=None, choices=sorted(RUSOLORN_SIZES), metavar="SIZES",
                   help="instead of the default workload: prefill and decode of a Rusolorn model (windowed attention "
                        "beside a gated delta rule, routed experts) at these layer sizes, beside the Kamedra model of "
                        "equal width, heads, active feed-forward size and layers, each with its stage times")
    p.add_argument("--metitar", default=None, choices=sorted(METITAR_SIZES), metavar="SIZES",
                   help="instead of the default workload: prefill and decode of a Metitar model (attention over a shared "
                        "latent, the HGRN2 recurrence, dense and routed feed-forwards) at these layer sizes, beside the "
                        "Rusolorn model of equal width, heads, experts and layers, each with its stage times")
    p.add_argument("--gizilorn", default=None, choices=sorted(GIZILORN_SIZES), metavar="SIZES",
                   help="instead of the default workload: prefill and decode of a Gizilorn model (several residual "
                        "streams, attention with mixed heads, windowed attention over a shared latent) at these layer "
                        "sizes, beside a Metitar model of equal width, latent and feed-forwards and a Qwen2.5-style model "
                        "of equal width, heads and window, each with its stage times")
    p.add_argument("--pusazen", default=None, choices=sorted(PUSAZEN_SIZES), metavar="SIZES",
                   help="instead of the default workload: prefill and decode of a Pusazen model (mLSTM, lightning attention, "
                        "chunked attention with capped scores and a sink, gated experts) at these layer sizes beside the "
                        "closest models of the engine")
    p.add_argument("--tomopel", default=None, choices=sorted(TOMOPEL_SIZES), metavar="SIZES",
                   help="instead of the default workload: prefill and decode of a Tomopel model (attention with a distance "
                        "bias beside Mamba-2, minGRU, ungated experts, several residual streams) at these layer sizes, "
                        "beside a Rusolorn model of equal width, heads, state, experts and layers and a Gizilorn model of "
                        "equal width, streams and dense feed-forward, each with its stage times")
    p.add_argument("--serving", type=int, default=0, metavar="REQUESTS",
                   help="also run this many requests (prompts of 128 to 2,048 tokens, 256 new tokens each) through "
                        "the scheduler with portions of 512, and report it under 'serving'")
    return p.parse_args()


def summarize_ms(samples_ms: list[float]) -> dict:
    """Mean, median, tail, spread and range of latency samples, as the reference summarises them
    (benchmarks/common.py:159-170)."""
    import numpy as np
    x = np.asarray(samples_ms, dtype=np.float64)
    return {"mean": round(float(x.mean()), 4), "median": round(float(np.percentile(x, 50)), 4),
            "p95": round(float(np.percentile(x, 95)), 4), "p99": round(float(np.percentile(x, 99)), 4),
            "std": round(float(x.std()), 4), "min": round(float(x.min()), 4), "max": round(float(x.max()), 4)}


def summarize_counts(samples: list[int]) -> dict:
    import numpy as np
    x = np.asarray(samples or [0], dtype=np.float64)
    return {"mean": round(float(x.mean()), 1), "median": float(np.percentile(x, 50)), "max": float(x.max())}


def environment(device) -> dict:
    """Where the numbers come from (the reference's collect_environment_metadata, benchmarks/common.py:231-251)."""
    import platform
    import subprocess

    import torch

    def git(*args: str) -> str | None:
        try:
            done = subprocess.run(["git", *args], cwd=ROOT, capture_output=True, text=True, timeout=10)
            return done.stdout.strip() if done.returncode == 0 else None
        except (OSError, subprocess.SubprocessError):
            return None

    props = torch.cuda.get_device_properties(device)
    dirty = git("status", "--porcelain")
    return {"git_sha": git("rev-parse", "HEAD"), "git_dirty": bool(dirty) if dirty is not None else None,
            "python_version": platform.python_version(), "platform": platform.platform(),
            "torch_version": torch.__version__, "hip_version": torch.version.hip,
            "device_name": props.name, "device_arch": getattr(props, "gcnArchName", None),
            "compute_units": props.multi_processor_count, "device_memory_gb": round(props.total_memory / 2**30, 1),
            "executable": sys.executable}


def measure_peaks(device) -> dict:
    """What this machine reaches on the two resources the step is bound by: streaming memory into the compute units
    (2 GiB, beyond every cache; the best of the read kernel's launch shapes) and bfloat16 matrix instructions on
    every SIMD."""
    import torch

    from somi_inference_amd.kernels import ops
    buffer = torch.empty(2 << 30, dtype=torch.uint8, device=device)
    buffer.zero_()

    def timed(fn, reps):
        fn()
        torch.cuda.synchronize()
        start, end = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        start.record()
        for _ in range(reps):
            fn()
        end.record()
        torch.cuda.synchronize()
        return start.elapsed_time(end) / reps / 1000.0
    shapes = {}
    for shape in ops.probe_stream_shapes():
        shapes[shape] = round((2 << 30) / 1e9 / timed(lambda: ops.probe_stream_read(buffer, shape), 5), 1)
    # matrix instructions on operands as a product has them, and on small integers (most bits zero: the clock under
    # matrix instructions goes with what the operands toggle, so this loop runs faster than any product can)
    flops = ops.probe_mfma(20000, device)
    mfma_s = timed(lambda: ops.probe_mfma(20000, device), 3)
    sparse_s = timed(lambda: ops.probe_mfma(20000, device, dense=False), 3)
    del buffer
    best = max(shapes, key=shapes.get)
    return {"stream_read_gbs": shapes[best], "stream_read_shape": best, "stream_read_by_shape": shapes,
            "mfma_bf16_tflops": round(flops / mfma_s / 1e12, 1),
            "mfma_bf16_tflops_small_integers": round(flops / sparse_s / 1e12, 1)}


def qwen2_config_dict(sizes: str, layers: int | None) -> dict:
    """The config.json of the Qwen2.5 layer sizes named ``sizes`` (with fewer layers if asked)."""
    full_layers, hidden, heads, kv_heads, head_dim, intermediate, eps, vocab, tied = LAYER_SIZES[sizes]
    return {"architectures": ["Qwen2ForCausalLM"], "model_type": "qwen2", "vocab_size": vocab, "hidden_size": hidden,
            "intermediate_size": intermediate, "num_hidden_layers": layers or full_layers,
            "num_attention_heads": heads, "num_key_value_heads": kv_heads, "head_dim": head_dim, "rope_theta": 1e6,
            "rms_norm_eps": eps, "tie_word_embeddings": tied, "max_position_embeddings": 32768,
            "hidden_act": "silu", "attention_bias": True}


class Workbench:
    """One model on the GPU with a cache pool, and the measurements that run on it.  The model comes from the
    registry by the architecture its config.json names; what a step costs is asked of the model's parts."""

    def __init__(self, config_dict: dict, *, dtype: str, seed: int, block_size: int, pool_tokens: int,
                 max_requests: int) -> None:
        import torch

        from somi_inference_amd.cache import CacheManager
        from somi_inference_amd.config.registry import config_from_dict
        from somi_inference_amd.models import make_runner, random_model
        from somi_inference_amd.sampling import Sampler, SamplingParams

        self.torch = torch
        _, self.config = config_from_dict(config_dict)
        self.config_dict = config_dict
        self.dtype, self.block_size = dtype, block_size
        self.device = torch.device("cuda:0")
        self.model = random_model(self.config, seed=seed, dtype=dtype, draw_on="device")
        self.num_blocks = (pool_tokens + block_size - 1) // block_size + max_requests + 1
        self.runner = make_runner(self.model, block_size=block_size, num_blocks=self.num_blocks, max_requests=max_requests + 1)
        self.sampler, self.greedy = Sampler(), SamplingParams(temperature=0.0)
        self.gen = torch.Generator().manual_seed(seed)
        self.vocab = self.model.vocab_size
        self.weight_bytes = self.model.step_weight_bytes()
        self.cache_bytes_per_token = CacheManager.page_bytes(self.model.cache_needs(), block_size,
                                                             self.model.runtime.dtype) / block_size

    def close(self) -> None:
        """Give the device memory back (weights, pool, captured graphs) before another model is built."""
        self.runner._graphs.clear()
        self.runner = self.model = self.sampler = None
        gc.collect()
        self.torch.cuda.empty_cache()

    def tokens(self, count: int) -> list[int]:
        return self.torch.randint(0, self.vocab, (count,), generator=self.gen).tolist()

    def decode_bytes(self, batch: int, mean_context: float) -> float:
        """What a decode step has to read: every weight once and the cache of the live requests."""
        return self.weight_bytes + batch * mean_context * self.cache_bytes_per_token

    # ------------------------------------------------------------------ decode
    def decode_run(self, batch: int, steps: int, warmup: int, context: int, portion: int = 2048) -> dict:
        """``batch`` requests whose prompts end ``warmup + steps`` tokens before the context length, run by the
        engine; times ``steps`` of its decode steps.  Every step is one scheduling decision, one model step for all
        requests and one sampling call, launched ahead of the device as generation does it.  The scheduler runs the
        prompts in portions and lets the requests that are done with theirs decode meanwhile, so a request has
        decoded some tokens before the timed steps begin (``mean_ctx`` says where the timed steps stood)."""
        from somi_inference_amd.engine import Engine, Request, Scheduler
        from somi_inference_amd.engine.engine import full_collections_deferred
        torch, runner = self.torch, self.runner
        scheduler = Scheduler(runner.cache, max_concurrent=batch, max_num_batched_tokens=max(portion, batch), chunk=portion)
        engine = Engine(runner, scheduler, self.sampler, eos_token_id=-1)
        prompt_len = context - (warmup + steps + 1)
        ramp = self.ramp(batch, context, portion)
        requests = [Request(f"b{batch}_{i}", self.tokens(prompt_len), ramp + warmup + steps + 8, self.greedy, seed=i)
                    for i in range(batch)]
        runner.capture_decode_graphs(batch, context + ramp)
        for request in requests:
            engine.add_request(request)
        with full_collections_deferred():          # as Engine.run() steps its requests
            while scheduler.waiting or any(r.num_computed < len(r.prompt_tokens) for r in requests):
                engine.step()
            for _ in range(warmup):
                engine.step()
            torch.cuda.synchronize()
            cached_before = sum(runner.cache.num_tokens(r.request_id) for r in requests)
            marks = [torch.cuda.Event(enable_timing=True) for _ in range(steps + 1)]
            marks[0].record()
            start = time.perf_counter()
            for i in range(steps):
                engine.step()
                marks[i + 1].record()
            torch.cuda.synchronize()
            seconds = time.perf_counter() - start
        cached_after = sum(runner.cache.num_tokens(r.request_id) for r in requests)
        assert cached_after - cached_before == batch * steps, "a timed step was not a decode step of every request"
        step_ms = [marks[i].elapsed_time(marks[i + 1]) for i in range(steps)]
        engine.abort(requests)
        mean_ctx = (cached_before + cached_after) / 2.0 / batch
        ms = 1000.0 * seconds / steps
        achieved = self.decode_bytes(batch, mean_ctx) / (ms / 1000.0) / 1e9
        return dict(tok_s=batch * steps / seconds, ms=ms, steps=steps, warmup=warmup, mean_ctx=mean_ctx,
                    step_ms=step_ms, run_ahead=engine.steps_run_ahead, achieved_gbs=achieved,
                    frac=achieved / HBM_PEAK_GBS)

    @staticmethod
    def ramp(batch: int, context: int, portion: int = 2048) -> int:
        """Tokens a request may decode while the others' prompts are still run, at most (beyond 128 requests the
        decoding tokens take a visible share of a step's tokens: a prompt then needs one portion more)."""
        return batch * ((context + portion - 1) // portion + (1 if batch > 128 else 0)) + 8

    @classmethod
    def pool_tokens(cls, batches, context: int, prefill_tokens: int = 0) -> int:
        most = max(batches)
        return max(most * (context + cls.ramp(most, context) + 32), prefill_tokens + 32)

    # ----------------------------------------------------------------- prefill
    def prefill_run(self, tokens: int, reps: int = 6) -> dict:
        from somi_inference_amd.engine import StepEntry
        torch, runner = self.torch, self.runner
        prompt = self.tokens(tokens)
        times = []
        for _ in range(reps):
            runner.begin("prefill")
            torch.cuda.synchronize()
            start = time.perf_counter()
            runner.step([StepEntry("prefill", prompt, [len(prompt) - 1])])
            torch.cuda.synchronize()
            times.append(time.perf_counter() - start)
            runner.end("prefill")
        times = sorted(times[1:])                     # the first run pays one-time set-up
        seconds = times[len(times) // 2]              # the median of the others
        flops = self.model.step_flops(tokens, tokens * (tokens + 1) // 2, 1)
        return {"value": round(tokens / seconds, 1), "tokens": tokens, "ms": round(seconds * 1000.0, 3),
                "frac": round(flops / seconds / PEAK_FLOPS[self.dtype], 4), "ms_min": round(times[0] * 1000.0, 3),
                "ms_max": round(times[-1] * 1000.0, 3), "tflop": round(flops / 1e12, 3)}

    # ----------------------------------------------------------------- serving
    def serving_run(self, count: int, max_concurrent: int, new_tokens: int = 256, chunk: int = 512,
                    budget: int = 2048, prompt_range: tuple[int, int] = (128, 2048)) -> dict:
        """Continuous batching through the engine's own scheduler: everything arrives at once, prompts of
        ``prompt_range`` tokens (128 to 2,048) are cut into portions of ``chunk`` under a budget of ``budget`` tokens a step, finished requests
        free their pages.  Reported as a whole, with what a step held (the reference reports a run with its arrival
        trace: benchmarks/bench_engine.py:181-283)."""
        from somi_inference_amd.engine import Engine, Request, Scheduler
        from somi_inference_amd.engine.engine import full_collections_deferred
        torch, runner = self.torch, self.runner
        shortest, longest = prompt_range
        lengths = torch.randint(shortest, longest + 1, (count,), generator=self.gen).tolist()
        per_request = (longest + new_tokens + self.block_size - 1) // self.block_size + 1
        concurrent = max(1, min(count, max_concurrent, self.num_blocks // per_request))
        scheduler = Scheduler(runner.cache, max_concurrent=concurrent, max_num_batched_tokens=budget, chunk=chunk)
        engine = Engine(runner, scheduler, self.sampler, eos_token_id=-1)
        requests = [Request(f"s{i}", self.tokens(n), new_tokens, self.greedy, seed=i) for i, n in enumerate(lengths)]
        # as LLM.warm_up() does it: the decode graphs that the requests will replay are captured before they arrive
        captured = runner.capture_decode_graphs(concurrent, longest + new_tokens)
        prompt_mix, decode_mix, live_mix = [], [], []
        torch.cuda.synchronize()
        start = time.perf_counter()
        for request in requests:
            engine.add_request(request)
        done = []
        with full_collections_deferred():
            while scheduler.has_unfinished():
                done.extend(engine.step())
                portions = engine.last_output.portions
                decoding = sum(1 for p in portions if p.start >= len(p.request.prompt_tokens))
                decode_mix.append(decoding)
                prompt_mix.append(sum(len(p.tokens) for p in portions) - decoding)
                live_mix.append(len(portions))
        done.extend(engine.run())                     # reads the last step's tokens
        torch.cuda.synchronize()
        seconds = time.perf_counter() - start
        generated = sum(len(r.output_tokens) for r in requests)
        assert all(len(r.output_tokens) == new_tokens for r in requests), "a request did not finish"
        return {"requests": len(requests), "prompt_tokens": sum(lengths), "generated_tokens": generated,
                "seconds": round(seconds, 3), "generated_tok_s": round(generated / seconds, 1),
                "total_tok_s": round((generated + sum(lengths)) / seconds, 1), "steps": engine.num_steps,
                "steps_run_ahead": engine.steps_run_ahead, "max_concurrent": concurrent,
                "preemptions": sum(r.num_preemptions for r in requests), "graphs_captured_ahead": captured,
                "step_mix": {"prompt_tokens": summarize_counts(prompt_mix), "decode_tokens": summarize_counts(decode_mix),
                             "live_requests": summarize_counts(live_mix)}}

    # ------------------------------------------------------------------ stages
    def stage_run(self, prefill_tokens: int, batch: int, context: int) -> dict:
        """Shares of the named stages in an eager prefill and in an eager decode step of ``batch`` requests at
        ``context`` tokens (captured graphs hold no stages, so the decode step is run without them)."""
        from somi_inference_amd.engine import StepEntry
        from somi_inference_amd.kernels import stages
        torch, runner = self.torch, self.runner
        out = {}
        prompt = self.tokens(prefill_tokens)
        for rep in range(2):                          # the second run is the one that counts
            runner.begin("stages")
            with stages.collect() as times:
                logits = runner.step([StepEntry("stages", prompt, [len(prompt) - 1])])
                self.sampler.sample(logits, self.greedy)
            out[f"prefill_{prefill_tokens}"] = times.summary()
            runner.end("stages")
        ids = [f"stage{i}" for i in range(batch)]
        for rid in ids:
            runner.begin(rid)
            runner.step([StepEntry(rid, self.tokens(context - 3), [])])
        graphs, runner.decode_graphs = runner.decode_graphs, False
        try:
            for rep in range(2):
                with stages.collect() as times:
                    logits = runner.step([StepEntry(rid, [1], [0]) for rid in ids])
                    self.sampler.sample(logits, [self.greedy] * batch)
                out[f"decode_b{batch}_eager"] = times.summary()
        finally:
            runner.decode_graphs = graphs
            for rid in ids:
                runner.end(rid)
        torch.cuda.synchronize()
        return out


def print_stage_tables(stage_times: dict) -> None:
    for what, rows in stage_times.items():
        total = sum(r["ms"] for r in rows.values())
        print(f"\n{what}: {total:.3f} ms in named stages", file=sys.stderr)
        print(f"  {'stage':<36}{'calls':>7}{'ms':>11}{'share':>9}", file=sys.stderr)
        for name, r in rows.items():
            print(f"  {name:<36}{r['calls']:>7}{r['ms']:>11.3f}{100 * r['share']:>8.1f}%", file=sys.stderr)


def config_block(bench: Workbench, label: str, batch: int, context: int, layers_of_config: int, mean_ctx: float) -> dict:
    data = bench.config.to_dict() if hasattr(bench.config, "to_dict") else dict(bench.config_dict)
    block = {"model": label, "global_batch": batch, "seq_len": context, "parallelism": "single GPU",
             "layers": data.get("num_hidden_layers"), "layers_of_config": layers_of_config}
    for key in SIZE_KEYS:
        if key in data and isinstance(data[key], (int, float, bool, str)):
            block[key] = data[key]
    block["block_size"] = bench.block_size
    block["mean_context"] = round(mean_ctx, 1)
    return block


def run_extras(args, started: float) -> dict:
    """Short measurements at the other configurations: each in a block of its own that reports an error instead of
    failing the line, none started once the run has taken ``--extras-budget`` seconds."""
    extras: dict = {}

    def within_budget(name: str) -> bool:
        if time.perf_counter() - started > args.extras_budget:
            extras[name] = {"skipped": f"the run had taken more than {args.extras_budget:.0f} s"}
            return False
        return True

    def point(run: dict) -> dict:
        return {"tok_s": round(run["tok_s"], 1), "ms": round(run["ms"], 4), "mean_ctx": round(run["mean_ctx"], 1),
                "frac": round(run["frac"], 4), "steps": run["steps"]}

    def attempt(name: str, fn) -> None:
        if not within_budget(name):
            return
        bench = None
        try:
            t0 = time.perf_counter()
            bench, result = fn()
            result["seconds_taken"] = round(time.perf_counter() - t0, 1)
            extras[name] = result
        except Exception as err:      # noqa: BLE001 - an extra must not fail the line
            extras[name] = {"error": f"{type(err).__name__}: {err}"[:300]}
        finally:
            import torch
            if bench is not None:
                bench.close()
            gc.collect()
            torch.cuda.empty_cache()

    def long_context():
        context = 32768
        bench = Workbench(qwen2_config_dict("7b", None), dtype=args.dtype, seed=args.seed, block_size=args.block_size,
                          pool_tokens=Workbench.pool_tokens([8], context), max_requests=8)
        return bench, {"sizes": "7b", "decode_b8": point(bench.decode_run(8, 16, 2, context))}

    def sizes_14b():
        bench = Workbench(qwen2_config_dict("14b", None), dtype=args.dtype, seed=args.seed, block_size=args.block_size,
                          pool_tokens=Workbench.pool_tokens([64], 4096), max_requests=64)
        result = {"sizes": "14b", "layers": 48}
        for batch in (8, 64):
            result[f"decode_b{batch}"] = point(bench.decode_run(batch, 16, 2, 4096))
        result["serving_32_requests"] = bench.serving_run(32, 32)
        return bench, result

    def sizes_32b():
        context = 8192
        bench = Workbench(qwen2_config_dict("32b", None), dtype=args.dtype, seed=args.seed, block_size=args.block_size,
                          pool_tokens=Workbench.pool_tokens([64], context), max_requests=64)
        result = {"sizes": "32b", "layers": 64, "prefill": bench.prefill_run(context, reps=3)}
        result["decode_b64"] = point(bench.decode_run(64, 16, 2, context))
        return bench, result

    attempt("long_context_7b", long_context)
    attempt("qwen2.5_14b", sizes_14b)
    attempt("qwen2.5_32b", sizes_32b)
    return extras


def run_kamedra(args) -> dict:
    """Prefill and decode of a Kamedra model beside the closest Qwen2.5-style model, with the stage times of both and
    what the attention and recurrence stages reach of the machine."""
    width, ff, heads, kv_heads, dim, vdim, r_heads, r_dim, r_vdim, rank, window, keep, vocab = KAMEDRA_SIZES[args.kamedra]
    batches, context, tokens = (8, 64), args.context, args.prefill_tokens
    out: dict = {}
    for label, config_dict in (("kamedra", kamedra_config_dict(args.kamedra)), ("closest", closest_config_dict(args.kamedra))):
        bench = Workbench(config_dict, dtype=args.dtype, seed=args.seed, block_size=args.block_size,
                          pool_tokens=Workbench.pool_tokens(batches, context, tokens), max_requests=max(batches))
        block: dict = {"prefill": {str(n): bench.prefill_run(n) for n in sorted({512, tokens})}}
        for batch in batches:
            run = bench.decode_run(batch, max(POINT_MIN_STEPS, args.steps // 2), max(2, args.warmup // 2), context)
            block[f"decode_b{batch}"] = {"tok_s": round(run["tok_s"], 1), "ms": round(run["ms"], 4),
                                        "mean_ctx": round(run["mean_ctx"], 1)}
        block["stages"] = bench.stage_run(tokens, batches[0], context)
        print_stage_tables(block["stages"])
        out[label] = block
        bench.close()
    # what the mixers' own kernels reach: matrix operations of a prefill's attention (both maps' scores and both
    # maps' weights times values over the visible pairs; causal pairs for the closest model) and of the recurrence
    bf16_peak = PEAK_FLOPS["bfloat16"]
    pairs_window = sum(min(p + 1, window + (keep if p >= window else 0)) for p in range(tokens))
    pairs_causal = tokens * (tokens + 1) // 2

    def stage_ms(block, run, name):
        return block["stages"][run].get(name, {}).get("ms", 0.0)
    run = f"prefill_{tokens}"
    k_ms, c_ms = stage_ms(out["kamedra"], run, "attention"), stage_ms(out["closest"], run, "attention")
    r_ms = stage_ms(out["kamedra"], run, "recurrence")
    k_flops = 2 * 4.0 * heads * (dim + vdim) * pairs_window           # two attention layers
    c_flops = 6 * 4.0 * heads * (2 * dim) * pairs_causal              # six attention layers
    r_flops = 4 * 4.0 * r_heads * r_dim * r_vdim * tokens             # four recurrent layers
    out["prefill_kernels"] = {
        "tokens": tokens,
        "kamedra_attention": {"ms": k_ms, "tflops": round(k_flops / 1e9 / max(k_ms, 1e-9), 2),
                              "frac_of_peak": round(k_flops / 1e3 / max(k_ms, 1e-9) / bf16_peak * 1e6, 5)},
        "closest_attention": {"ms": c_ms, "tflops": round(c_flops / 1e9 / max(c_ms, 1e-9), 2),
                              "frac_of_peak": round(c_flops / 1e3 / max(c_ms, 1e-9) / bf16_peak * 1e6, 5)},
        "kamedra_recurrence": {"ms": r_ms, "tflops": round(r_flops / 1e9 / max(r_ms, 1e-9), 3)},
    }
    # a decode step's attention reads the visible keys and values; its recurrence reads and writes the states
    run = f"decode_b{batches[0]}_eager"
    k_ms, c_ms = stage_ms(out["kamedra"], run, "attention"), stage_ms(out["closest"], run, "attention")
    r_ms = stage_ms(out["kamedra"], run, "recurrence")
    seen = min(context, window + keep)
    k_bytes = 2 * batches[0] * seen * kv_heads * (2 * dim + vdim) * 2.0
    c_bytes = 6 * batches[0] * context * kv_heads * (2 * 2 * dim) * 2.0
    r_bytes = 4 * batches[0] * r_heads * r_dim * r_vdim * 4.0 * 2
    out["decode_kernels"] = {
        "batch": batches[0], "context": context,
        "kamedra_attention": {"ms": k_ms, "gbs": round(k_bytes / 1e6 / max(k_ms, 1e-9), 1)},
        "closest_attention": {"ms": c_ms, "gbs": round(c_bytes / 1e6 / max(c_ms, 1e-9), 1)},
        "kamedra_recurrence": {"ms": r_ms, "gbs": round(r_bytes / 1e6 / max(r_ms, 1e-9), 1)},
    }
    return out


def run_rusolorn(args) -> dict:
    """Prefill and decode of a Rusolorn model beside the closest Kamedra model, with the stage times of both and what
    the attention, recurrence and feed-forward stages reach of the machine."""
    (width, heads, kv_heads, dim, window, r_heads, r_groups, r_dim, r_vdim, taps, experts, top, groups, keep, ff, shared,
     side, vocab) = RUSOLORN_SIZES[args.rusolorn]
    batches, context, tokens = (8, 64), args.context, args.prefill_tokens
    out: dict = {}
    for label, config_dict in (("rusolorn", rusolorn_config_dict(args.rusolorn)),
                               ("closest", rusolorn_closest_config_dict(args.rusolorn))):
        bench = Workbench(config_dict, dtype=args.dtype, seed=args.seed, block_size=args.block_size,
                          pool_tokens=Workbench.pool_tokens(batches, context, tokens), max_requests=max(batches))
        block: dict = {"prefill": {str(n): bench.prefill_run(n) for n in sorted({512, tokens})}}
        for batch in batches:
            run = bench.decode_run(batch, max(POINT_MIN_STEPS, args.steps // 2), max(2, args.warmup // 2), context)
            block[f"decode_b{batch}"] = {"tok_s": round(run["tok_s"], 1), "ms": round(run["ms"], 4),
                                        "mean_ctx": round(run["mean_ctx"], 1)}
        block["stages"] = bench.stage_run(tokens, batches[0], context)
        print_stage_tables(block["stages"])
        out[label] = block
        bench.close()
    bf16_peak = PEAK_FLOPS["bfloat16"]
    pairs = sum(min(p + 1, window) for p in range(tokens))

    def stage_ms(block, run, *names):
        return sum(block["stages"][run].get(name, {}).get("ms", 0.0) for name in names)

    def rate(flops, ms):
        return {"ms": round(ms, 4), "tflops": round(flops / 1e9 / max(ms, 1e-9), 2),
                "frac_of_peak": round(flops / 1e3 / max(ms, 1e-9) / bf16_peak * 1e6, 5)}
    run, layers, half = f"prefill_{tokens}", RUSOLORN_LAYERS, RUSOLORN_LAYERS // 2
    out["prefill_kernels"] = {
        "tokens": tokens,
        # scores and weights times values over the visible pairs (the closest model: two maps of half the key size)
        "rusolorn_attention": rate(layers * 4.0 * heads * dim * pairs, stage_ms(out["rusolorn"], run, "attention")),
        "closest_attention": rate(half * 4.0 * heads * (dim // 2 + dim) * pairs, stage_ms(out["closest"], run, "attention")),
        # per token and head: three passes over the state here (two products, one update), two in the closest model
        "rusolorn_recurrence": rate(layers * 6.0 * r_heads * r_dim * r_vdim * tokens, stage_ms(out["rusolorn"], run, "recurrence")),
        "closest_recurrence": rate(half * 4.0 * r_heads * r_dim * r_vdim * tokens, stage_ms(out["closest"], run, "recurrence")),
        # the routed experts' three matrices over the pairs, against the dense feed-forward's products
        "rusolorn_experts": rate(layers * 6.0 * tokens * top * ff * width,
                                 stage_ms(out["rusolorn"], run, "experts gate_up", "experts down")),
        "closest_feed_forward": rate(layers * 6.0 * tokens * (top * ff + shared) * width,
                                     stage_ms(out["closest"], run, "gate_up", "down")),
        "rusolorn_router": {"ms": round(stage_ms(out["rusolorn"], run, "router"), 4)},
    }
    run = f"decode_b{batches[0]}_eager"

    def stream(bytes_, ms):
        return {"ms": round(ms, 4), "gbs": round(bytes_ / 1e6 / max(ms, 1e-9), 1)}
    seen = min(context, window)
    used = min(experts, batches[0] * top)          # experts a step touches at most
    out["decode_kernels"] = {
        "batch": batches[0], "context": context,
        "rusolorn_attention": stream(layers * batches[0] * seen * kv_heads * 2 * dim * 2.0, stage_ms(out["rusolorn"], run, "attention")),
        "closest_attention": stream(half * batches[0] * seen * kv_heads * (dim + dim) * 2.0, stage_ms(out["closest"], run, "attention")),
        "rusolorn_recurrence": stream(layers * batches[0] * r_heads * r_dim * r_vdim * 4.0 * 2, stage_ms(out["rusolorn"], run, "recurrence")),
        "closest_recurrence": stream(half * batches[0] * r_heads * r_dim * r_vdim * 4.0 * 2, stage_ms(out["closest"], run, "recurrence")),
        "rusolorn_experts": stream(layers * used * 3.0 * ff * width * 2.0,
                                   stage_ms(out["rusolorn"], run, "experts gate_up", "experts down")),
        "closest_feed_forward": stream(layers * 3.0 * (top * ff + shared) * width * 2.0,
                                       stage_ms(out["closest"], run, "gate_up", "down")),
    }
    return out


def run_metitar(args) -> dict:
    """Prefill and decode of a Metitar model beside the closest Rusolorn model, with the stage times of both and what
    the attention, recurrence and feed-forward stages reach of the machine."""
    (width, heads, dim, rot, vdim, rank, q_rank, r_heads, r_dim, r_vdim, taps, experts, top, ff, shared, dense_ff, side,
     vocab) = METITAR_SIZES[args.metitar]
    batches, context, tokens = (8, 64), args.context, args.prefill_tokens
    out: dict = {}
    for label, config_dict in (("metitar", metitar_config_dict(args.metitar)),
                               ("closest", metitar_closest_config_dict(args.metitar))):
        bench = Workbench(config_dict, dtype=args.dtype, seed=args.seed, block_size=args.block_size,
                          pool_tokens=Workbench.pool_tokens(batches, context, tokens), max_requests=max(batches))
        block: dict = {"prefill": {str(n): bench.prefill_run(n) for n in sorted({512, tokens})}}
        for batch in batches:
            run = bench.decode_run(batch, max(POINT_MIN_STEPS, args.steps // 2), max(2, args.warmup // 2), context)
            block[f"decode_b{batch}"] = {"tok_s": round(run["tok_s"], 1), "ms": round(run["ms"], 4),
                                        "mean_ctx": round(run["mean_ctx"], 1)}
        block["stages"] = bench.stage_run(tokens, batches[0], context)
        print_stage_tables(block["stages"])
        out[label] = block
        bench.close()
    bf16_peak = PEAK_FLOPS["bfloat16"]
    pairs = tokens * (tokens + 1) // 2

    def stage_ms(block, run, *names):
        return sum(block["stages"][run].get(name, {}).get("ms", 0.0) for name in names)

    def rate(flops, ms):
        return {"ms": round(ms, 4), "tflops": round(flops / 1e9 / max(ms, 1e-9), 2),
                "frac_of_peak": round(flops / 1e3 / max(ms, 1e-9) / bf16_peak * 1e6, 5)}
    run, layers = f"prefill_{tokens}", METITAR_LAYERS
    attention_layers, recurrent_layers, expert_layers, dense_layers = 3, 3, 3, 3
    out["prefill_kernels"] = {
        "tokens": tokens,
        # scores over the latent and the shared key part, weights times the latent, over the visible pairs
        "metitar_attention": rate(attention_layers * 2.0 * heads * (2 * rank + rot) * pairs, stage_ms(out["metitar"], run, "attention")),
        "closest_attention": rate(layers * 4.0 * heads * dim * pairs, stage_ms(out["closest"], run, "attention")),
        # the per-head maps on either side of the attention (no like kernel in the closest model)
        "metitar_head_maps": rate(attention_layers * 2.0 * tokens * heads * rank * (dim + vdim),
                                  stage_ms(out["metitar"], run, "queries to the latent's side", "values from the latent")),
        # per token and head: two passes over the state here (update, product), three in the closest model
        "metitar_recurrence": rate(recurrent_layers * 4.0 * r_heads * r_dim * r_vdim * tokens, stage_ms(out["metitar"], run, "recurrence")),
        "closest_recurrence": rate(layers * 6.0 * r_heads * r_dim * r_vdim * tokens, stage_ms(out["closest"], run, "recurrence")),
        "metitar_experts": rate(expert_layers * 6.0 * tokens * top * ff * width,
                                stage_ms(out["metitar"], run, "experts gate_up", "experts down")),
        "closest_experts": rate(layers * 6.0 * tokens * top * ff * width,
                                stage_ms(out["closest"], run, "experts gate_up", "experts down")),
        "metitar_dense": rate(dense_layers * 4.0 * tokens * dense_ff * width, stage_ms(out["metitar"], run, "up", "down")),
        "metitar_router": {"ms": round(stage_ms(out["metitar"], run, "router"), 4)},
        "closest_router": {"ms": round(stage_ms(out["closest"], run, "router"), 4)},
    }
    run = f"decode_b{batches[0]}_eager"

    def stream(bytes_, ms):
        return {"ms": round(ms, 4), "gbs": round(bytes_ / 1e6 / max(ms, 1e-9), 1)}
    used = min(experts, batches[0] * top)          # experts a step touches at most
    out["decode_kernels"] = {
        "batch": batches[0], "context": context,
        # one kept vector a token for all heads, against keys and values for every key/value head
        "metitar_attention": stream(attention_layers * batches[0] * context * (rank + rot) * 2.0, stage_ms(out["metitar"], run, "attention")),
        "closest_attention": stream(layers * batches[0] * context * (heads // 4) * 2 * dim * 2.0, stage_ms(out["closest"], run, "attention")),
        "metitar_recurrence": stream(recurrent_layers * batches[0] * r_heads * r_dim * r_vdim * 4.0 * 2, stage_ms(out["metitar"], run, "recurrence")),
        "closest_recurrence": stream(layers * batches[0] * r_heads * r_dim * r_vdim * 4.0 * 2, stage_ms(out["closest"], run, "recurrence")),
        "metitar_experts": stream(expert_layers * used * 3.0 * ff * width * 2.0,
                                  stage_ms(out["metitar"], run, "experts gate_up", "experts down")),
        "closest_experts": stream(layers * used * 3.0 * ff * width * 2.0,
                                  stage_ms(out["closest"], run, "experts gate_up", "experts down")),
    }
    return out


def run_gizilorn(args) -> dict:
    """Prefill and decode of a Gizilorn model beside the closest models the engine had, with the stage times of all
    three and what the attention kernels, the dense products and the kernels between the sublayers reach of the machine."""
    (width, streams, heads, kv_heads, dim, window, l_heads, l_dim, rot, vdim, rank, l_window, ff, vocab) = GIZILORN_SIZES[args.gizilorn]
    batches, context, tokens = (8, 64), args.context, args.prefill_tokens
    out: dict = {}
    for label, config_dict in (("gizilorn", gizilorn_config_dict(args.gizilorn)),
                               ("closest", gizilorn_closest_config_dict(args.gizilorn)),
                               ("closest_attention", gizilorn_closest_attention_config_dict(args.gizilorn))):
        bench = Workbench(config_dict, dtype=args.dtype, seed=args.seed, block_size=args.block_size,
                          pool_tokens=Workbench.pool_tokens(batches, context, tokens), max_requests=max(batches))
        block: dict = {"prefill": {str(n): bench.prefill_run(n) for n in sorted({512, tokens})}}
        for batch in batches:
            run = bench.decode_run(batch, max(POINT_MIN_STEPS, args.steps // 2), max(2, args.warmup // 2), context)
            block[f"decode_b{batch}"] = {"tok_s": round(run["tok_s"], 1), "ms": round(run["ms"], 4),
                                        "mean_ctx": round(run["mean_ctx"], 1)}
        block["stages"] = bench.stage_run(tokens, batches[0], context)
        print_stage_tables(block["stages"])
        out[label] = block
        bench.close()
    bf16_peak = PEAK_FLOPS["bfloat16"]

    def pairs_of(size):
        return sum(min(p + 1, size) for p in range(tokens))

    def stage_ms(block, run, *names):
        return sum(block["stages"][run].get(name, {}).get("ms", 0.0) for name in names)

    def rate(flops, ms):
        return {"ms": round(ms, 4), "tflops": round(flops / 1e9 / max(ms, 1e-9), 2),
                "frac_of_peak": round(flops / 1e3 / max(ms, 1e-9) / bf16_peak * 1e6, 5)}

    def stream(bytes_, ms):
        return {"ms": round(ms, 4), "gbs": round(bytes_ / 1e6 / max(ms, 1e-9), 1)}
    run, layers, half = f"prefill_{tokens}", GIZILORN_LAYERS, GIZILORN_LAYERS // 2
    out["prefill_kernels"] = {
        "tokens": tokens,
        # useful work over the visible pairs: scores once and weights times values once (the kernel computes the scores
        # twice, mixes the heads' weights and multiplies the weights in two halves)
        "gizilorn_attention": rate(half * 2.0 * heads * (dim + dim) * pairs_of(window),
                                   stage_ms(out["gizilorn"], run, "mixed attention")),
        "closest_attention": rate(layers * 4.0 * heads * dim * pairs_of(window), stage_ms(out["closest_attention"], run, "attention")),
        "closest_latent_attention": rate(layers * 2.0 * l_heads * (2 * rank + rot) * pairs_of(tokens),
                                         stage_ms(out["closest"], run, "attention")),
        "gizilorn_dense": rate(layers * 4.0 * tokens * ff * width, stage_ms(out["gizilorn"], run, "up", "down")),
        "closest_dense": rate(layers * 4.0 * tokens * ff * width, stage_ms(out["closest"], run, "up", "down")),
        # between the sublayers: every stream read and written in float32, the sublayer's rows read, the normed rows written
        "gizilorn_streams": stream(layers * 2.0 * tokens * width * (8.0 * streams + 4 + 2),
                                   stage_ms(out["gizilorn"], run, "residual add, norm")),
        "closest_output_norm": stream(layers * 2.0 * tokens * width * (8.0 + 4 + 2),
                                      stage_ms(out["closest"], run, "output norm, residual add")),
    }
    run = f"decode_b{batches[0]}_eager"
    out["decode_kernels"] = {
        "batch": batches[0], "context": context,
        "gizilorn_attention": stream(half * batches[0] * min(context, window) * kv_heads * 2 * dim * 2.0,
                                     stage_ms(out["gizilorn"], run, "mixed attention")),
        "closest_attention": stream(layers * batches[0] * min(context, window) * kv_heads * 2 * dim * 2.0,
                                    stage_ms(out["closest_attention"], run, "attention")),
        "closest_latent_attention": stream(layers * batches[0] * context * (rank + rot) * 2.0,
                                           stage_ms(out["closest"], run, "attention")),
        "gizilorn_streams": stream(layers * 2.0 * batches[0] * width * (8.0 * streams + 4 + 2),
                                   stage_ms(out["gizilorn"], run, "residual add, norm")),
    }
    for kernels, tokens_or_batch, seen in ((out["prefill_kernels"], None, pairs_of(l_window)),
                                           (out["decode_kernels"], batches[0], None)):
        name = "prefill_%d" % tokens if tokens_or_batch is None else run
        ms = stage_ms(out["gizilorn"], name, "attention")
        if tokens_or_batch is None:
            kernels["gizilorn_latent_attention"] = rate(half * 2.0 * l_heads * (2 * rank + rot) * seen, ms)
        else:
            kernels["gizilorn_latent_attention"] = stream(half * tokens_or_batch * min(context, l_window) * (rank + rot) * 2.0, ms)
    return out


def run_tomopel(args) -> dict:
    """Prefill and decode of a Tomopel model beside the closest models the engine had, with the stage times of all three
    and what the attention, recurrence, expert and stream kernels reach of the machine."""
    (width, streams, heads, kv_heads, dim, r_heads, r_vdim, state, groups, taps, gru, experts, top, ff, shared, dense_ff,
     vocab) = TOMOPEL_SIZES[args.tomopel]
    batches, context, tokens = (8, 64), args.context, args.prefill_tokens
    out: dict = {}
    for label, config_dict in (("tomopel", tomopel_config_dict(args.tomopel)), ("closest", tomopel_closest_config_dict(args.tomopel)),
                               ("closest_streams", tomopel_closest_streams_config_dict(args.tomopel))):
        bench = Workbench(config_dict, dtype=args.dtype, seed=args.seed, block_size=args.block_size,
                          pool_tokens=Workbench.pool_tokens(batches, context, tokens), max_requests=max(batches))
        block: dict = {"prefill": {str(n): bench.prefill_run(n) for n in sorted({512, tokens})}}
        for batch in batches:
            run = bench.decode_run(batch, max(POINT_MIN_STEPS, args.steps // 2), max(2, args.warmup // 2), context)
            block[f"decode_b{batch}"] = {"tok_s": round(run["tok_s"], 1), "ms": round(run["ms"], 4),
                                        "mean_ctx": round(run["mean_ctx"], 1)}
        block["stages"] = bench.stage_run(tokens, batches[0], context)
        print_stage_tables(block["stages"])
        out[label] = block
        bench.close()
    bf16_peak = PEAK_FLOPS["bfloat16"]
    pairs = tokens * (tokens + 1) // 2
    layers, mixed, routed = TOMOPEL_LAYERS, TOMOPEL_PARALLEL, TOMOPEL_LAYERS - 1

    def stage_ms(block, run, *names):
        return sum(block["stages"][run].get(name, {}).get("ms", 0.0) for name in names)

    def rate(flops, ms):
        return {"ms": round(ms, 4), "tflops": round(flops / 1e9 / max(ms, 1e-9), 2),
                "frac_of_peak": round(flops / 1e3 / max(ms, 1e-9) / bf16_peak * 1e6, 5)}

    def stream(bytes_, ms):
        return {"ms": round(ms, 4), "gbs": round(bytes_ / 1e6 / max(ms, 1e-9), 1)}
    run = f"prefill_{tokens}"
    inner = r_heads * r_vdim
    channels = inner + 2 * groups * state
    delta_heads = inner * state // (128 * 128)
    out["prefill_kernels"] = {
        "tokens": tokens,
        "tomopel_attention": rate(mixed * 4.0 * heads * dim * pairs, stage_ms(out["tomopel"], run, "attention")),
        "closest_attention": rate(layers * 4.0 * heads * dim * pairs, stage_ms(out["closest"], run, "attention")),
        # per token and element of the state: its update and its product with C here (two passes), three in the closest model
        "tomopel_recurrence": rate(mixed * 4.0 * inner * state * tokens, stage_ms(out["tomopel"], run, "recurrence")),
        "closest_recurrence": rate(layers * 6.0 * delta_heads * 128 * 128 * tokens, stage_ms(out["closest"], run, "recurrence")),
        # three float32 rows read, one row written in the compute dtype
        "tomopel_gated_recurrence": stream(tokens * gru * (12.0 + 2), stage_ms(out["tomopel"], run, "gated recurrence")),
        # x, B and C read and written in float32 (the closest model's stage reads bfloat16 rows and norms q and k as well)
        "tomopel_convolution": stream(mixed * tokens * channels * 8.0, stage_ms(out["tomopel"], run, "convolution")),
        "closest_convolution": stream(layers * tokens * 2 * delta_heads * 128 * 6.0, stage_ms(out["closest"], run, "convolution, unit norms")),
        # y and z read in float32, the normed rows written
        "tomopel_gate_norm": stream(mixed * tokens * inner * 10.0, stage_ms(out["tomopel"], run, "gate, norm")),
        "closest_gate_norm": stream(layers * tokens * delta_heads * 128 * 8.0, stage_ms(out["closest"], run, "norm, gate")),
        # the q/k/v sums read, q, k and v written (the closest model's rows are bfloat16)
        "tomopel_head_norms": stream(mixed * tokens * (heads + 2 * kv_heads) * dim * 6.0, stage_ms(out["tomopel"], run, "head norms, k/v into pages")),
        "closest_qk_norm": stream(layers * tokens * ((heads + kv_heads) * dim * 4.0 + kv_heads * dim * 2.0), stage_ms(out["closest"], run, "q/k norm, k/v into pages")),
        "tomopel_experts": rate(routed * 4.0 * tokens * top * ff * width, stage_ms(out["tomopel"], run, "experts up", "experts down")),
        "closest_experts": rate(layers * 6.0 * tokens * top * ff * width, stage_ms(out["closest"], run, "experts gate_up", "experts down")),
        "tomopel_products": rate(mixed * 2.0 * tokens * width * ((heads + 2 * kv_heads) * dim + heads + inner + channels + r_heads + heads * dim + inner)
                                 + 2.0 * tokens * width * 4 * gru + 6.0 * tokens * width * dense_ff,
                                 stage_ms(out["tomopel"], run, "inputs", "o", "z/x/g", "gate_up", "down")),
        "closest_products": rate(layers * 2.0 * tokens * width * ((2 * heads + kv_heads) * dim + 4 * delta_heads * 128),
                                 stage_ms(out["closest"], run, "q/k/v", "q/k/v/g", "o")),
        "tomopel_streams": stream(layers * 2.0 * tokens * width * (8.0 * streams + 4 + 2), stage_ms(out["tomopel"], run, "residual add, norm")),
        "closest_streams": stream(layers * 2.0 * tokens * width * (8.0 * streams + 4 + 2), stage_ms(out["closest_streams"], run, "residual add, norm")),
        "tomopel_router": {"ms": round(stage_ms(out["tomopel"], run, "router"), 4)},
        "closest_router": {"ms": round(stage_ms(out["closest"], run, "router"), 4)},
    }
    run = f"decode_b{batches[0]}_eager"
    used = min(experts, batches[0] * top)          # experts a step touches at most
    out["decode_kernels"] = {
        "batch": batches[0], "context": context,
        "tomopel_attention": stream(mixed * batches[0] * context * kv_heads * 2 * dim * 2.0, stage_ms(out["tomopel"], run, "attention")),
        "closest_attention": stream(layers * batches[0] * context * kv_heads * 2 * dim * 2.0, stage_ms(out["closest"], run, "attention")),
        "tomopel_recurrence": stream(mixed * batches[0] * inner * state * 8.0, stage_ms(out["tomopel"], run, "recurrence")),
        "closest_recurrence": stream(layers * batches[0] * delta_heads * 128 * 128 * 8.0, stage_ms(out["closest"], run, "recurrence")),
        "tomopel_experts": stream(routed * used * 2.0 * ff * width * 2.0, stage_ms(out["tomopel"], run, "experts up", "experts down")),
        "closest_experts": stream(layers * used * 3.0 * ff * width * 2.0, stage_ms(out["closest"], run, "experts gate_up", "experts down")),
        "tomopel_streams": stream(layers * 2.0 * batches[0] * width * (8.0 * streams + 4 + 2), stage_ms(out["tomopel"], run, "residual add, norm")),
        "closest_streams": stream(layers * 2.0 * batches[0] * width * (8.0 * streams + 4 + 2), stage_ms(out["closest_streams"], run, "residual add, norm")),
    }
    return out


def run_pusazen(args) -> dict:
    """Prefill and decode of a Pusazen model beside the closest models the engine had (Tomopel: the recurrence, the attention
    and what normed heads take; Rusolorn: gated experts; Metitar: an ungated dense feed-forward and a norm behind a sublayer),
    with the stage times of all four and what the kernels reach of the machine."""
    (width, m_heads, m_dim, m_vdim, l_heads, l_dim, l_vdim, heads, kv_heads, dim, chunk, experts, top, ff, shared, dense_ff,
     vocab) = PUSAZEN_SIZES[args.pusazen]
    (_, t_streams, t_heads, t_kv, t_dim, r_heads, r_vdim, r_state, *_) = TOMOPEL_SIZES[args.pusazen]
    batches, context, tokens = (8, 64), args.context, args.prefill_tokens
    out: dict = {}
    for label, config_dict in (("pusazen", pusazen_config_dict(args.pusazen)), ("closest", tomopel_config_dict(args.pusazen)),
                               ("closest_experts", tomopel_closest_config_dict(args.pusazen)),
                               ("closest_dense", pusazen_closest_dense_config_dict(args.pusazen))):
        bench = Workbench(config_dict, dtype=args.dtype, seed=args.seed, block_size=args.block_size,
                          pool_tokens=Workbench.pool_tokens(batches, context, tokens), max_requests=max(batches))
        block: dict = {"prefill": {str(n): bench.prefill_run(n) for n in sorted({512, tokens})}}
        for batch in batches:
            run = bench.decode_run(batch, max(POINT_MIN_STEPS, args.steps // 2), max(2, args.warmup // 2), context)
            block[f"decode_b{batch}"] = {"tok_s": round(run["tok_s"], 1), "ms": round(run["ms"], 4),
                                        "mean_ctx": round(run["mean_ctx"], 1)}
        block["stages"] = bench.stage_run(tokens, batches[0], context)
        print_stage_tables(block["stages"])
        out[label] = block
        bench.close()
    bf16_peak = PEAK_FLOPS["bfloat16"]
    count = PUSAZEN_LAYERS
    layers, routed = sum(count.values()), sum(count.values()) - 1
    theirs, t_mixed = TOMOPEL_LAYERS, TOMOPEL_PARALLEL

    def stage_ms(label, run, *names):
        return sum(out[label]["stages"][run].get(name, {}).get("ms", 0.0) for name in names)

    def rate(flops, ms):
        return {"ms": round(ms, 4), "tflops": round(flops / 1e9 / max(ms, 1e-9), 2),
                "frac_of_peak": round(flops / 1e3 / max(ms, 1e-9) / bf16_peak * 1e6, 5)}

    def stream(bytes_, ms):
        return {"ms": round(ms, 4), "gbs": round(bytes_ / 1e6 / max(ms, 1e-9), 1)}
    pairs = sum(p % chunk + 1 for p in range(tokens))
    m_state, l_state, inner = m_heads * m_dim * (m_vdim + 1), l_heads * l_dim * l_vdim, r_heads * r_vdim
    state = count["mlstm"] * m_state + count["lightning"] * l_state
    mixed = count["mlstm"] * m_heads * m_vdim + count["lightning"] * l_heads * l_vdim
    run = f"prefill_{tokens}"
    out["prefill_kernels"] = {
        "tokens": tokens,
        "pusazen_attention": rate(count["attention"] * 4.0 * heads * dim * pairs, stage_ms("pusazen", run, "attention")),
        "closest_attention": rate(t_mixed * 4.0 * t_heads * t_dim * tokens * (tokens + 1) / 2, stage_ms("closest", run, "attention")),
        # per token and element of the state: its update and its product with q (or C)
        "pusazen_recurrence": rate(4.0 * state * tokens, stage_ms("pusazen", run, "recurrence")),
        "closest_recurrence": rate(t_mixed * 4.0 * inner * r_state * tokens, stage_ms("closest", run, "recurrence")),
        "pusazen_gates": {"ms": round(stage_ms("pusazen", run, "gates"), 4)},
        # q, k and v read and written in float32; x, B and C through a convolution
        "pusazen_input_activation": stream(count["lightning"] * tokens * l_heads * (2 * l_dim + l_vdim) * 8.0, stage_ms("pusazen", run, "input activation")),
        "closest_convolution": stream(t_mixed * tokens * (inner + 2 * r_state) * 8.0, stage_ms("closest", run, "convolution")),
        # y and the gate read in float32, the normed rows written
        "pusazen_norm_gate": stream(tokens * mixed * 10.0, stage_ms("pusazen", run, "norm, gate")),
        "closest_gate_norm": stream(t_mixed * tokens * inner * 10.0, stage_ms("closest", run, "gate, norm")),
        # the q/k/v sums read in float32, q, k and v written
        "pusazen_qk_norm": stream(count["attention"] * tokens * (heads + 2 * kv_heads) * dim * 6.0,
                                  stage_ms("pusazen", run, "q/k norm, position encoding, k/v into pages")),
        "closest_head_norms": stream(t_mixed * tokens * (t_heads + 2 * t_kv) * t_dim * 6.0, stage_ms("closest", run, "head norms, k/v into pages")),
        "pusazen_experts": rate(routed * 6.0 * tokens * top * ff * width, stage_ms("pusazen", run, "experts gate_up", "experts down")),
        "closest_experts": rate(theirs * 6.0 * tokens * top * ff * width, stage_ms("closest_experts", run, "experts gate_up", "experts down")),
        "pusazen_shared": rate(routed * 6.0 * tokens * shared * width, stage_ms("pusazen", run, "shared gate_up", "shared activation", "shared down")),
        "closest_shared": rate(theirs * 6.0 * tokens * shared * width, stage_ms("closest_experts", run, "shared gate_up", "shared activation", "shared down")),
        "pusazen_router": {"ms_a_layer": round(stage_ms("pusazen", run, "router") / routed, 4)},
        "closest_router": {"ms_a_layer": round(stage_ms("closest_experts", run, "router") / theirs, 4)},
        "pusazen_dense": rate(4.0 * tokens * dense_ff * width, stage_ms("pusazen", run, "up", "down", "activation")),
        "closest_dense": rate(6 * 4.0 * tokens * dense_ff * width, stage_ms("closest_dense", run, "up", "down", "activation")),
        "pusazen_mixer_products": rate(2.0 * tokens * width * (
            count["mlstm"] * m_heads * (2 * m_dim + 3 * m_vdim + 2) + count["lightning"] * l_heads * (2 * l_dim + 3 * l_vdim)
            + count["attention"] * (2 * heads + 2 * kv_heads) * dim), stage_ms("pusazen", run, "q/k/v/g/gates", "q/k/v/g", "q/k/v", "o")),
        "closest_mixer_products": rate(theirs * 2.0 * tokens * width * 4 * l_heads * l_dim, stage_ms("closest_dense", run, "q/f/v", "o")),
        # the stream read and written in float32, the sublayer's rows read, the new rows written once more in 16 bits
        "pusazen_sum_norm": stream(2 * layers * tokens * width * (8.0 + 4 + 2), stage_ms("pusazen", run, "sum, norm")),
        "closest_output_norm": stream(12 * tokens * width * (8.0 + 4 + 2), stage_ms("closest_dense", run, "output norm, residual add")),
    }
    run = f"decode_b{batches[0]}_eager"
    used = min(experts, batches[0] * top)          # experts a step touches at most
    seen = (context - 1) % chunk + 1
    out["decode_kernels"] = {
        "batch": batches[0], "context": context,
        "pusazen_attention": stream(count["attention"] * batches[0] * seen * kv_heads * 2 * dim * 2.0, stage_ms("pusazen", run, "attention")),
        "closest_attention": stream(t_mixed * batches[0] * context * t_kv * 2 * t_dim * 2.0, stage_ms("closest", run, "attention")),
        "pusazen_recurrence": stream(batches[0] * state * 8.0, stage_ms("pusazen", run, "recurrence")),
        "closest_recurrence": stream(t_mixed * batches[0] * inner * r_state * 8.0, stage_ms("closest", run, "recurrence")),
        "pusazen_experts": stream(routed * used * 3.0 * ff * width * 2.0, stage_ms("pusazen", run, "experts gate_up", "experts down")),
        "closest_experts": stream(theirs * used * 3.0 * ff * width * 2.0, stage_ms("closest_experts", run, "experts gate_up", "experts down")),
        "pusazen_dense": stream(2.0 * dense_ff * width * 2.0, stage_ms("pusazen", run, "up", "down", "activation")),
        "closest_dense": stream(6 * 2.0 * dense_ff * width * 2.0, stage_ms("closest_dense", run, "up", "down", "activation")),
        "pusazen_sum_norm": {"ms_a_layer": round(stage_ms("pusazen", run, "sum, norm") / layers, 4)},
        "closest_output_norm": {"ms_a_layer": round(stage_ms("closest_dense", run, "output norm, residual add") / 6, 4)},
    }
    return out


def main() -> int:
    args = parse_args()
    world = int(os.environ.get("WORLD_SIZE", "1"))
    if args.gpus != 1 or world != 1:
        if int(os.environ.get("RANK", "0")) == 0:
            print(f"bench.py: this engine runs on one GPU; --gpus {args.gpus} (WORLD_SIZE {world}) is not supported")
        return 2
    started = time.perf_counter()
    if args.kamedra:
        line = {"metric": f"Kamedra at {args.kamedra} layer sizes beside the closest Qwen2.5-style model: prefill and decode",
                "unit": "tokens/s", "n_gpus": 1, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
                "data": "synthetic: seeded random weights, seeded uniform token ids", "sizes": args.kamedra}
        line.update(run_kamedra(args))
        line["value"] = line["kamedra"][f"decode_b8"]["tok_s"]
        line["seconds_total"] = round(time.perf_counter() - started, 1)
        print(json.dumps(line))
        return 0

    if args.pusazen:
        line = {"metric": f"Pusazen at {args.pusazen} layer sizes beside the closest Tomopel, Rusolorn and Metitar models: prefill and decode",
                "unit": "tokens/s", "n_gpus": 1, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
                "data": "synthetic: seeded random weights, seeded uniform token ids", "sizes": args.pusazen}
        line.update(run_pusazen(args))
        line["value"] = line["pusazen"]["decode_b8"]["tok_s"]
        line["seconds_total"] = round(time.perf_counter() - started, 1)
        print(json.dumps(line))
        return 0

    if args.tomopel:
        line = {"metric": f"Tomopel at {args.tomopel} layer sizes beside the closest Rusolorn and Gizilorn models: prefill and decode",
                "unit": "tokens/s", "n_gpus": 1, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
                "data": "synthetic: seeded random weights, seeded uniform token ids", "sizes": args.tomopel}
        line.update(run_tomopel(args))
        line["value"] = line["tomopel"]["decode_b8"]["tok_s"]
        line["seconds_total"] = round(time.perf_counter() - started, 1)
        print(json.dumps(line))
        return 0

    if args.gizilorn:
        line = {"metric": f"Gizilorn at {args.gizilorn} layer sizes beside the closest Metitar and Qwen2.5-style models: prefill and decode",
                "unit": "tokens/s", "n_gpus": 1, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
                "data": "synthetic: seeded random weights, seeded uniform token ids", "sizes": args.gizilorn}
        line.update(run_gizilorn(args))
        line["value"] = line["gizilorn"]["decode_b8"]["tok_s"]
        line["seconds_total"] = round(time.perf_counter() - started, 1)
        print(json.dumps(line))
        return 0

    if args.metitar:
        line = {"metric": f"Metitar at {args.metitar} layer sizes beside the closest Rusolorn model: prefill and decode",
                "unit": "tokens/s", "n_gpus": 1, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
                "data": "synthetic: seeded random weights, seeded uniform token ids", "sizes": args.metitar}
        line.update(run_metitar(args))
        line["value"] = line["metitar"]["decode_b8"]["tok_s"]
        line["seconds_total"] = round(time.perf_counter() - started, 1)
        print(json.dumps(line))
        return 0

    if args.rusolorn:
        line = {"metric": f"Rusolorn at {args.rusolorn} layer sizes beside the closest Kamedra model: prefill and decode",
                "unit": "tokens/s", "n_gpus": 1, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
                "data": "synthetic: seeded random weights, seeded uniform token ids", "sizes": args.rusolorn}
        line.update(run_rusolorn(args))
        line["value"] = line["rusolorn"]["decode_b8"]["tok_s"]
        line["seconds_total"] = round(time.perf_counter() - started, 1)
        print(json.dumps(line))
        return 0

    import torch

    if args.config_json:
        with open(args.config_json, "r", encoding="utf-8") as handle:
            config_dict = json.load(handle)
        layers_of_config = int(config_dict.get("num_hidden_layers", 0))
        if args.layers:
            config_dict["num_hidden_layers"] = args.layers
        label = f"{(config_dict.get('architectures') or ['?'])[0]} from {os.path.basename(os.path.abspath(args.config_json))} (random weights)"
        name = label
    else:
        layers_of_config = LAYER_SIZES[args.sizes][0]
        config_dict = qwen2_config_dict(args.sizes, args.layers)
        label = f"Qwen2.5-{args.sizes.upper()} layer sizes (random weights)"
        name = f"Qwen2.5-{args.sizes.upper()} layer sizes"
    torch.manual_seed(args.seed)
    batches = [args.batch] if args.no_points else sorted({1, args.batch, *POINT_BATCHES})
    bench = Workbench(config_dict, dtype=args.dtype, seed=args.seed, block_size=args.block_size,
                      pool_tokens=Workbench.pool_tokens(batches, args.context, args.prefill_tokens),
                      max_requests=max(batches))

    results = {}
    for batch in batches:
        steps = args.steps if batch == args.batch else max(POINT_MIN_STEPS, args.steps // (2 if batch <= 64 else 4))
        warmup = args.warmup if batch == args.batch else max(2, args.warmup // 2)
        results[batch] = bench.decode_run(batch, steps, warmup, args.context)
    main_run = results[args.batch]
    peaks = None if args.no_peaks else measure_peaks(bench.device)

    prefill = None
    if not args.no_prefill:
        prefill = bench.prefill_run(args.prefill_tokens)
        if peaks is not None and args.dtype == "bfloat16":
            prefill["frac_of_measured_mfma"] = round(prefill["tflop"] * 1e12 / (prefill["ms"] / 1000.0)
                                                     / (peaks["mfma_bf16_tflops"] * 1e12), 4)
    serving = bench.serving_run(args.serving, max(batches)) if args.serving > 0 else None
    stage_times = bench.stage_run(args.prefill_tokens, args.batch, args.context) if args.stages else None

    roofline = {"bound": "hbm", "achieved": round(main_run["achieved_gbs"], 1), "peak": HBM_PEAK_GBS, "unit": "GB/s",
                "frac": round(main_run["frac"], 4)}
    if peaks is not None:
        roofline["measured_peak"] = peaks["stream_read_gbs"]
        roofline["frac_of_measured"] = round(main_run["achieved_gbs"] / peaks["stream_read_gbs"], 4)
    line = {
        "metric": f"decode tok/s at batch {args.batch}, {name} "
                  f"(plus prefill tok/s at {args.prefill_tokens:,} tokens, batch 1/64/96/128/256 points)",
        "value": round(main_run["tok_s"], 2), "unit": "tokens/s", "n_gpus": 1,
        "steps": main_run["steps"], "warmup": main_run["warmup"], "ms_per_step": round(main_run["ms"], 4),
        "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
        "data": "synthetic: seeded random N(0,0.02) weights, seeded uniform token ids; prompts run and tokens decoded "
                "by the engine's own generation loop",
        "config": config_block(bench, label, args.batch, args.context, layers_of_config, main_run["mean_ctx"]),
        "roofline": roofline,
        "latency_ms": summarize_ms(main_run["step_ms"]),
        "points": {f"decode_b{b}": round(r["tok_s"], 2) for b, r in results.items() if b in POINT_BATCHES},
        "point_details": {f"decode_b{b}": {"ms": round(r["ms"], 4), "mean_ctx": round(r["mean_ctx"], 1),
                                           "frac": round(r["frac"], 4), "steps": r["steps"]}
                          for b, r in results.items() if b in POINT_BATCHES},
    }
    if prefill is not None:
        line["prefill"] = prefill
    if serving is not None:
        line["serving"] = serving
    if peaks is not None:
        line["measured_peaks"] = peaks
    if stage_times is not None:
        line["stages"] = stage_times
        print_stage_tables(stage_times)
    line["environment"] = environment(bench.device)
    default_run = not args.config_json and args.sizes == "7b" and not args.layers and not args.no_points
    if default_run and not args.no_extras:
        bench.close()
        line["extras"] = run_extras(args, started)
    line["seconds_total"] = round(time.perf_counter() - started, 1)
    text = json.dumps(line)
    print(text)
    if args.output_file:
        os.makedirs(os.path.dirname(os.path.abspath(args.output_file)), exist_ok=True)
        with open(args.output_file, "a", encoding="utf-8") as handle:      # appended, as the reference's runs are
            handle.write(text + "\n")
    return 0


if __name__ == "__main__":
    sys.exit(main())
