"""The Pusazen decoder as a plan: layers that norm the residual sum (the stream weighed by a constant plus a sublayer's scaled
output) and whose sublayers read the stream itself; the mixer is mLSTM, lightning attention, or grouped-query attention in
chunks with a norm over the whole projections, a partial rotation, capped scores and a sink; the feed-forward is a dense one
with a squared relu or a mixture of gated experts (a biased router, a shared expert behind a gate); an untied head whose
logits are scaled.

Tensor names: ``embed``, ``final.norm``, ``head``, and per layer ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.ls1``, ``l<i>.ls2``,
``l<i>.mix.{q,k,v,g,o,norm,i,i.b,f,f.b}`` or ``l<i>.mix.{q,k,v,g,o,norm}`` or ``l<i>.mix.{q,k,v,o,q.norm,k.norm,sink}``,
``l<i>.mlp.{up,down}`` or ``l<i>.mlp.{router,router.b,e<j>.gate,e<j>.up,e<j>.down,shared.gate,shared.up,shared.down,
shared.sg}``; no name carries a ``.weight`` suffix.
"""

from __future__ import annotations

from ..config.pusazen import PusazenConfig, PusazenDense
from ..config.registry import register_architecture
from ..parts.base import PartSpec
from .plan import LayerSpec, ModelPlan

ATTENTION_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm", "sink": "sink"}
BLOCK_NAMES = {"mixer_norm": "", "mixer": "mix", "ffn_norm": "", "feed_forward": "mlp", "mixer_scale": "ls1", "ffn_scale": "ls2"}


def pusazen_plan(config: PusazenConfig) -> ModelPlan:
    def norm(tensor: str) -> PartSpec:
        return PartSpec("rmsnorm", {"hidden_size": config.width, "eps": config.norm_eps, "tensor": tensor})

    layers = []
    for index, layer in enumerate(config.layers):
        m, mlp = layer.mixer, layer.mlp
        if layer.type == "mlstm":
            mixer = PartSpec("mlstm", {"hidden_size": config.width, "num_heads": m.heads, "key_dim": m.dim, "value_dim": m.vdim,
                                       "gate_cap": m.gate_cap, "eps": config.norm_eps, "suffix": ""})
        elif layer.type == "lightning":
            mixer = PartSpec("lightning_attention", {"hidden_size": config.width, "num_heads": m.heads, "key_dim": m.dim,
                                                     "value_dim": m.vdim, "decay": m.decay, "eps": config.norm_eps, "suffix": ""})
        else:
            position = (PartSpec("none", {}) if m.rot_base is None else
                        PartSpec("rotary", {"head_dim": m.dim, "theta": m.rot_base, "rotary_dim": m.rot_dims, "double": True}))
            mixer = PartSpec("gqa_attention", {
                "hidden_size": config.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim,
                "value_dim": m.vdim, "position": position, "qkv_bias": False, "scale": m.scale, "qk_norm": "projection",
                "norm_eps": config.norm_eps, "chunk": m.chunk, "softcap": m.softcap, "sink": True, "names": ATTENTION_NAMES,
                "suffix": ""})
        if mlp is None:
            feed_forward = None
        elif isinstance(mlp, PusazenDense):
            feed_forward = PartSpec("activated", {"hidden_size": config.width, "intermediate_size": mlp.ff,
                                                  "activation": "squared_relu", "bias": False, "suffix": ""})
        else:
            feed_forward = PartSpec("routed_experts", {
                "hidden_size": config.width, "num_experts": mlp.experts, "top": mlp.top, "expert_size": mlp.ff,
                "shared_size": mlp.shared_ff, "alpha": 1.0, "shift": 0.0, "router_bias": True,
                "shared_gate": mlp.shared_ff is not None, "suffix": ""})
        block = PartSpec("sum_norm", {
            "mixer": mixer, "feed_forward": feed_forward, "mixer_norm": norm("norm1"),
            "ffn_norm": None if feed_forward is None else norm("norm2"), "width": config.width, "alpha": config.alpha,
            "names": BLOCK_NAMES})
        layers.append(LayerSpec(f"l{index}", block))
    return ModelPlan(
        embedding=PartSpec("token_embedding", {"vocab_size": config.vocab, "hidden_size": config.width, "tensor": "embed"}),
        embedding_prefix="",
        layers=tuple(layers),
        final_norm=norm("norm"),
        final_norm_prefix="final",
        head=PartSpec("lm_head", {"vocab_size": config.vocab, "hidden_size": config.width, "tied": False, "tensor": "head",
                                  "scale": config.logit_scale}),
        head_prefix="",
        vocab_size=config.vocab,
    )


register_architecture(PusazenConfig.architecture, PusazenConfig, pusazen_plan, replace=True)
