"""The Tomopel decoder as a plan: pre-norm layers around several residual streams (hyper-connections) with a scaled
residual add; the mixer is grouped-query attention (heads normed one by one, a learned distance bias, a query temperature
and a gate a head) beside Mamba-2, their outputs added with a scale each, or a minGRU; the feed-forward is a dense gated
one or a mixture of experts (squared relu, softmax scores with a correction for the choice, a shared expert); a scaled
embedding and an untied head; norm weights stored around zero.

Tensor names: ``embed``, ``final.norm``, ``head``, and per layer ``l<i>.norm1``, ``l<i>.norm2``,
``l<i>.mix.left.{q,k,v,g,o,q.norm,k.norm,rel}``, ``l<i>.mix.right.{in,conv,conv.b,dt_bias,A_log,D,norm,o}`` or
``l<i>.mix.{z,z.b,x,x.b,g,o}``, ``l<i>.mlp.{gate,up,down}`` or ``l<i>.mlp.{router,correction,e<j>.up,e<j>.down,
shared.up,shared.down}``, ``l<i>.hc1.{in,out,mix}`` and ``l<i>.hc2.{in,out,mix}``; no name carries a ``.weight`` suffix.
"""

from __future__ import annotations

from ..config.registry import register_architecture
from ..config.tomopel import TomopelConfig, TomopelDense
from ..parts.base import PartSpec
from .plan import LayerSpec, ModelPlan

BLOCK_NAMES = {"mixer_norm": "", "mixer": "mix", "ffn_norm": "", "feed_forward": "mlp", "mixer_streams": "hc1",
               "ffn_streams": "hc2"}
DENSE_NAMES = {"gate": "gate", "up": "up", "down": "down"}


def tomopel_plan(config: TomopelConfig) -> ModelPlan:
    def norm(tensor: str) -> PartSpec:
        return PartSpec("rmsnorm", {"hidden_size": config.width, "eps": config.norm_eps, "tensor": tensor, "around_one": True})

    layers = []
    for index, layer in enumerate(config.layers):
        m = layer.mixer
        if layer.type == "parallel":
            left, right = m.left, m.right
            mixer = PartSpec("parallel", {
                "hidden_size": config.width, "join": "scaled_sum", "left_scale": m.left_scale, "right_scale": m.right_scale,
                "left": PartSpec("biased_attention", {
                    "hidden_size": config.width, "num_heads": left.heads, "num_kv_heads": left.kv_heads, "dim": left.dim,
                    "value_dim": left.vdim, "scale": left.scale, "eps": config.norm_eps, "bias_max": left.bias_max,
                    "buckets": left.buckets, "suffix": "",
                    "temperature": None if left.temp_coef is None else (left.temp_coef, left.temp_every)}),
                "right": PartSpec("mamba2", {
                    "hidden_size": config.width, "num_heads": right.heads, "num_groups": right.groups,
                    "state_dim": right.state, "value_dim": right.vdim, "taps": right.conv, "norm_groups": right.norm_groups,
                    "eps": config.norm_eps, "suffix": ""})})
        else:
            mixer = PartSpec("min_gru", {"hidden_size": config.width, "width": m.width, "suffix": ""})
        mlp = layer.mlp
        if mlp is None:
            feed_forward = None
        elif isinstance(mlp, TomopelDense):
            feed_forward = PartSpec("swiglu", {"hidden_size": config.width, "intermediate_size": mlp.ff, "names": DENSE_NAMES,
                                               "suffix": ""})
        else:
            feed_forward = PartSpec("routed_experts", {
                "hidden_size": config.width, "num_experts": mlp.experts, "top": mlp.top, "expert_size": mlp.ff,
                "shared_size": mlp.shared_ff, "unit": "squared_relu", "correction": True, "suffix": ""})
        block = PartSpec("hyper_connections", {
            "mixer": mixer, "feed_forward": feed_forward, "mixer_norm": norm("norm1"),
            "ffn_norm": None if feed_forward is None else norm("norm2"), "streams": config.streams or 1,
            "connections": config.streams is not None, "residual_mult": config.residual_mult, "names": BLOCK_NAMES})
        layers.append(LayerSpec(f"l{index}", block))
    return ModelPlan(
        embedding=PartSpec("token_embedding", {"vocab_size": config.vocab, "hidden_size": config.width, "tensor": "embed",
                                               "scale": config.embedding_scale}),
        embedding_prefix="",
        layers=tuple(layers),
        final_norm=norm("norm"),
        final_norm_prefix="final",
        head=PartSpec("lm_head", {"vocab_size": config.vocab, "hidden_size": config.width, "tied": False, "tensor": "head"}),
        head_prefix="",
        vocab_size=config.vocab,
    )


register_architecture(TomopelConfig.architecture, TomopelConfig, tomopel_plan, replace=True)
