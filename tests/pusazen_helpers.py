"""Small Pusazen configurations for the tests and their model folders."""

import os

from somi_inference_amd.config import (PusazenAttention, PusazenConfig, PusazenDense, PusazenExperts, PusazenLayer,
                                       PusazenLightning, PusazenMLSTM)


def mlstm(heads, dim, vdim, cap, mlp=None):
    return PusazenLayer("mlstm", PusazenMLSTM(heads, dim, vdim, cap), mlp)


def lightning(dim, vdim, decay, mlp=None):
    return PusazenLayer("lightning", PusazenLightning(len(decay), dim, vdim, tuple(decay)), mlp)


def attention(heads, kv, dim, vdim, scale, cap, base, dims, chunk, mlp=None):
    return PusazenLayer("attention", PusazenAttention(heads, kv, dim, vdim, scale, cap, base, dims, chunk), mlp)


# A: several query heads a key/value head, value sizes unlike key sizes, chunks that end inside pages, a partial rotation,
#    experts with and without a shared one, a layer without a feed-forward, an odd number of heads (padded input rows).
# B: attention first; head size 64 (the 32 x 32 tile kernel) with the whole head rotated, chunks of whole pages; constants of
#    one (alpha, the logits' scale) and decays of one and of almost nothing.
# C: odd sizes everywhere, a width that is no multiple of 8, pages of 4 tokens, chunks of 5, every expert chosen.
# D: head size 128 with one key/value head, a cap that bites, one expert a token, keys of more than 64 channels.
PUSAZEN = {
    "A": dict(seed=41, block_size=8, config=PusazenConfig(
        vocab=299, width=96, norm_eps=1e-6, alpha=2.5, logit_scale=1.5, layers=(
            mlstm(3, 20, 28, 12.0, PusazenExperts(6, 2, 40, 24)),
            attention(6, 2, 24, 40, 0.3, 30.0, 10000.0, 12, 45, PusazenDense(56)),
            lightning(16, 24, (0.5, 0.9, 0.97), PusazenExperts(5, 3, 32)),
            mlstm(2, 32, 16, 9.0, None),
        ))),
    "B": dict(seed=42, block_size=16, config=PusazenConfig(
        vocab=131, width=64, norm_eps=1e-5, alpha=1.0, logit_scale=1.0, layers=(
            attention(4, 4, 64, 64, 0.2, 50.0, 500.0, 64, 96, PusazenDense(40)),
            lightning(64, 64, (1.0, 0.02), PusazenExperts(4, 2, 24, 56)),
            mlstm(2, 64, 64, 15.0, PusazenDense(72)),
        ))),
    "C": dict(seed=43, block_size=4, config=PusazenConfig(
        vocab=97, width=76, norm_eps=1e-6, alpha=3.7, logit_scale=0.6, layers=(
            lightning(9, 7, (0.3, 0.99, 0.8, 0.6, 0.95), PusazenDense(36)),
            attention(3, 1, 20, 33, 0.4, 12.0, 2000.0, 2, 5, PusazenExperts(3, 3, 20, 12)),
            mlstm(1, 13, 50, 4.0, PusazenDense(21)),
            attention(5, 5, 10, 6, 0.7, 20.0, 300.0, 10, 61, None),
        ))),
    "D": dict(seed=44, block_size=16, config=PusazenConfig(
        vocab=211, width=72, norm_eps=1e-6, alpha=2.0, logit_scale=3.0, layers=(
            mlstm(5, 8, 12, 20.0, PusazenDense(48)),
            attention(5, 1, 128, 128, 0.25, 2.5, 40000.0, 96, 130, PusazenExperts(9, 1, 48, 8)),
            mlstm(2, 100, 36, 6.0, PusazenExperts(7, 2, 24)),
            lightning(80, 40, (0.999, 0.4), PusazenDense(56)),
        ))),
}


def write_pusazen(name: str, folder: str, peaky: bool = False) -> str:
    """The model folder of configuration ``name``.  Random matrices this small would leave the sublayers without a say
    beside the stream, so they are widened, routers too, so that they decide something.  ``peaky``: the query norms' weights
    are widened, so that attention scores spread over several units and single keys stand out."""
    from safetensors.torch import load_file, save_file

    from somi_inference_amd.weights import write_random_model
    write_random_model(folder, PUSAZEN[name]["config"], seed=PUSAZEN[name]["seed"])
    path = os.path.join(folder, "model.safetensors")
    tensors = load_file(path)
    for key, tensor in list(tensors.items()):
        factor = 1.0
        if tensor.dim() == 2 and (".mlp." in key or ".mix." in key):
            factor = 6.0
        if key.endswith((".router", ".router.b")):
            factor = 8.0
        if key.endswith((".mix.i", ".mix.f", ".shared.sg")):
            factor = 10.0
        if key == "embed":
            factor = 50.0
        if key == "head":
            factor = 5.0
        if peaky and key.endswith(".q.norm"):
            factor = 3.0
        tensors[key] = (tensor.float() * factor).to(tensor.dtype)
    save_file(tensors, path)
    return folder


def load_plain(folder: str, dtype=None):
    import torch

    from plain import pusazen_plain
    return pusazen_plain.load_folder(folder, dtype or torch.float32)
