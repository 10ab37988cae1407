"""Small Tomopel configurations for the tests and their model folders."""

import os

import torch

from somi_inference_amd.config import (TomopelAttention, TomopelConfig, TomopelDense, TomopelExperts, TomopelLayer,
                                       TomopelMamba2, TomopelMinGRU, TomopelParallel)


def parallel(heads, kv, dim, vdim, scale, bias_max, buckets, temp, right, left_scale=1.0, right_scale=1.0, mlp=None):
    """``temp``: (coef, every) or None; ``right``: (heads, vdim, state, groups, conv, norm_groups)."""
    left = TomopelAttention(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=scale, bias_max=bias_max, buckets=buckets,
                            temp_coef=None if temp is None else temp[0], temp_every=1 if temp is None else temp[1])
    return TomopelLayer("parallel", TomopelParallel(left, TomopelMamba2(*right), left_scale, right_scale), mlp)


def mingru(width, mlp=None):
    return TomopelLayer("mingru", TomopelMinGRU(width), mlp)


# A: three streams; query heads a key/value head that are no power of two, value size unlike the key size, both mixers'
#    scales unlike one, two groups of B and C and two normed parts, experts with and without a shared one (of another
#    size), a layer without a feed-forward, a temperature that moves every few positions.
# B: ONE stream that still has connection tensors; head size 64 (the 32 x 32 tile kernel); bucket edges that fall exactly
#    on whole distances; one tap; no temperature; a residual multiplier and an embedding scale of one; minGRU first.
# C: no connection tensors at all (the plain residual sum, scaled); odd sizes everywhere, a width that is no multiple of
#    8, pages of 4 tokens, an odd number of buckets, nine taps, every expert chosen, only dense and routed in turn.
# D: four streams; head size 128 with one key/value head; a bias that reaches past several pages and key tiles; a state
#    of more than 64 rows; one expert a token.
TOMOPEL = {
    "A": dict(seed=31, block_size=8, config=TomopelConfig(
        vocab=301, width=96, norm_eps=1e-6, embedding_scale=2.0, residual_mult=0.6, streams=3, layers=(
            parallel(6, 2, 24, 16, 0.35, 60, 10, (0.7, 7), (4, 12, 20, 2, 4, 2), 0.7, 1.3, TomopelExperts(6, 2, 40, 24)),
            mingru(72, TomopelDense(64)),
            parallel(4, 4, 16, 40, 0.5, 33, 8, (0.3, 16), (2, 24, 16, 1, 2, 1), 1.5, 0.4, None),
            mingru(40, TomopelExperts(5, 3, 32)),
        ))),
    "B": dict(seed=32, block_size=16, config=TomopelConfig(
        vocab=130, width=64, norm_eps=1e-5, embedding_scale=1.0, residual_mult=1.0, streams=1, layers=(
            mingru(33, TomopelDense(40)),
            parallel(4, 2, 64, 64, 0.2, 128, 16, None, (3, 16, 33, 3, 1, 3), 1.0, 1.0, TomopelExperts(4, 2, 24, 56)),
        ))),
    "C": dict(seed=33, block_size=4, config=TomopelConfig(
        vocab=97, width=76, norm_eps=1e-6, embedding_scale=3.0, residual_mult=0.45, streams=None, layers=(
            parallel(3, 1, 20, 33, 0.4, 19, 7, (1.1, 3), (5, 7, 9, 5, 9, 1), 0.8, 0.9, TomopelDense(36)),
            parallel(5, 5, 10, 6, 0.7, 300, 4, (0.2, 100), (6, 10, 70, 2, 3, 4), 0.5, 1.1, TomopelExperts(3, 3, 20, 12)),
            mingru(50, None),
        ))),
    "D": dict(seed=34, block_size=16, config=TomopelConfig(
        vocab=211, width=72, norm_eps=1e-6, embedding_scale=0.7, residual_mult=0.8, streams=4, layers=(
            parallel(5, 1, 128, 128, 0.12, 190, 24, (0.5, 40), (2, 40, 130, 1, 4, 1), 0.9, 0.6, TomopelExperts(9, 1, 48, 8)),
            parallel(2, 1, 48, 32, 0.3, 90, 12, (0.4, 25), (4, 8, 32, 1, 4, 2), 0.6, 1.0, TomopelDense(56)),
        ))),
}


def write_tomopel(name: str, folder: str, peaky: bool = False) -> str:
    """The model folder of configuration ``name``.  Random matrices this small would leave the sublayers without a say
    beside the streams, so they are widened, routers too, so that they decide something.  ``peaky``: the query norms'
    weights are widened, so that attention scores spread over several units and single keys stand out."""
    from safetensors.torch import load_file, save_file

    from somi_inference_amd.weights import write_random_model
    write_random_model(folder, TOMOPEL[name]["config"], seed=TOMOPEL[name]["seed"])
    path = os.path.join(folder, "model.safetensors")
    tensors = load_file(path)
    for key, tensor in list(tensors.items()):
        factor = 1.0
        if tensor.dim() == 2 and (".mlp." in key or ".mix." in key) and not key.endswith((".rel", ".conv")):
            factor = 6.0
        if key.endswith(".router"):
            factor = 8.0
        if key.endswith(".correction"):
            factor = 10.0
        if key == "embed":
            factor = 20.0
        if peaky and key.endswith(".q.norm"):
            factor = 3.0
        if peaky and key.endswith(".rel"):
            factor = 2.0
        tensors[key] = (tensor.float() * factor).to(tensor.dtype)
    save_file(tensors, path)
    return folder


def load_plain(folder: str, dtype=torch.float32):
    from plain import tomopel_plain
    return tomopel_plain.load_folder(folder, dtype)
