"""The Pusazen configuration, its plan and what the plan asks of the cache manager (no GPU)."""

import copy

import pytest
import torch

from plain import pusazen_plain as plain
from pusazen_helpers import PUSAZEN
from somi_inference_amd.config import ConfigError, PusazenConfig, config_from_dict
from somi_inference_amd.models import DecoderModel, collect_weight_specs, pusazen_plan
from somi_inference_amd.parts import (ActivatedFF, CompositeSpec, FixedStateSpec, PagedKVSpec, PartSpec, ResidualStream, RoutedExperts,
                                      Runtime, build_part)


def raw(name="A"):
    return PUSAZEN[name]["config"].to_dict()


@pytest.mark.parametrize("name", list(PUSAZEN))
def test_config_round_trip_and_registry(name):
    config = PUSAZEN[name]["config"]
    arch, again = config_from_dict(config.to_dict())
    assert arch.name == "Pusazen" and again == config and isinstance(again, PusazenConfig)


def test_keys_a_model_may_leave_out():
    data = raw("A")
    del data["layers"][0]["mlp"]["shared"], data["layers"][1]["mixer"]["kv_heads"]
    for key in ("mask", "rot", "softcap"):
        del data["layers"][1]["mixer"][key]
    config = PusazenConfig.from_dict(data)
    mixer = config.layers[1].mixer
    assert mixer.kv_heads == mixer.heads == 6 and mixer.chunk is None and mixer.softcap is None and mixer.rot_base is None
    assert config.layers[0].mlp.shared_ff is None and config.layers[3].mlp is None
    assert PusazenConfig.from_dict(config.to_dict()) == config
    specs = {s.name for s in collect_weight_specs(pusazen_plan(config))}
    assert "l0.mlp.shared.up" not in specs and "l0.mlp.shared.sg" not in specs and "l3.mlp.up" not in specs and "l3.ls2" not in specs


@pytest.mark.parametrize("change,word", [
    (lambda d: d["layers"][0]["mixer"].pop("gate_cap"), "gate_cap"),
    (lambda d: d["layers"][0]["mixer"].update(gate_cap=0.0), "gate_cap"),
    (lambda d: d["layers"][1]["mixer"].update(kv_heads=4), "kv_heads"),
    (lambda d: d["layers"][1]["mixer"].update(scale=0.0), "scale"),
    (lambda d: d["layers"][1]["mixer"].update(softcap=-1.0), "softcap"),
    (lambda d: d["layers"][1]["mixer"]["rot"].update(dims=7), "rot.dims"),
    (lambda d: d["layers"][1]["mixer"]["rot"].update(dims=26), "rot.dims"),
    (lambda d: d["layers"][1]["mixer"]["mask"].update(size=0), "size"),
    (lambda d: d["layers"][2]["mixer"].update(decay=[0.5]), "decay"),
    (lambda d: d["layers"][2]["mixer"].update(decay="slow"), "decay"),
    (lambda d: d["layers"][2].update(type="recurrence"), "type"),
    (lambda d: d["layers"][0]["mlp"]["router"].update(top=7), "top"),
    (lambda d: d["layers"][0]["mlp"].update(kind="sparse"), "kind"),
    (lambda d: d.pop("vocab"), "vocab"),
])
def test_what_is_refused(change, word):
    data = copy.deepcopy(raw("A"))
    change(data)
    with pytest.raises(ConfigError, match=word):
        PusazenConfig.from_dict(data)


def test_tensor_names_and_shapes():
    specs = {s.name: s for s in collect_weight_specs(pusazen_plan(PUSAZEN["A"]["config"]))}
    assert specs["embed"].shape == (299, 96) and specs["head"].shape == (299, 96) and specs["final.norm"].shape == (96,)
    assert specs["l0.mix.q"].shape == specs["l0.mix.k"].shape == (60, 96) and specs["l0.mix.v"].shape == (84, 96)
    assert specs["l0.mix.i"].shape == (3, 96) and specs["l0.mix.f.b"].shape == (3,) and specs["l0.mix.norm"].shape == (84,)
    assert specs["l0.mix.g"].shape == (84, 96) and specs["l0.mix.o"].shape == (96, 84)
    assert specs["l1.mix.q"].shape == (144, 96) and specs["l1.mix.k"].shape == (48, 96) and specs["l1.mix.v"].shape == (80, 96)
    assert specs["l1.mix.q.norm"].shape == (144,) and specs["l1.mix.k.norm"].shape == (48,) and specs["l1.mix.sink"].shape == (6,)
    assert specs["l1.mix.o"].shape == (96, 240) and specs["l1.mlp.up"].shape == (56, 96) and "l1.mlp.act" not in specs
    assert specs["l2.mix.q"].shape == (48, 96) and specs["l2.mix.v"].shape == (72, 96) and "l2.mix.i" not in specs
    assert specs["l0.mlp.router.b"].shape == (6,) and specs["l0.mlp.e5.gate"].shape == (40, 96) and specs["l0.mlp.shared.sg"].shape == (1, 96)
    assert "l2.mlp.shared.up" not in specs and specs["l0.ls1"].shape == specs["l0.ls2"].shape == (96,)
    assert "l3.ls1" in specs and "l3.ls2" not in specs and "l3.norm2" not in specs
    assert not any(name.endswith((".weight", ".bias")) for name in specs)


def test_what_a_layer_keeps():
    model = DecoderModel(pusazen_plan(PUSAZEN["A"]["config"]), Runtime(torch.float32, torch.device("cpu")))
    first, second, third, _ = model.cache_needs()
    assert isinstance(first, CompositeSpec) and isinstance(second, PagedKVSpec) and isinstance(third, FixedStateSpec)
    kept = dict(first.parts)
    assert kept["state"].shape == (3, 29, 20) and kept["top"].shape == (3,)           # the normaliser is one column more
    assert kept["state"].dtype == kept["top"].dtype == third.dtype == torch.float32
    assert second.chunk == 45 and second.window is None and second.num_kv_heads == 2 and second.head_dim == 48
    assert third.shape == (3, 24, 16)
    assert model.entry_splits() == [8] and model.graph_safe()


def test_sizes_no_kernel_takes_are_refused_when_the_part_is_built():
    attention = dict(hidden_size=16, num_heads=4, num_kv_heads=2, head_dim=16, position=PartSpec("none", {}), qkv_bias=False)
    for change in (dict(num_kv_heads=3), dict(value_dim=300, qk_norm="projection"), dict(softcap=-2.0), dict(value_dim=8)):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("gqa_attention", {**attention, **change}), prefix="m")
    mlstm = dict(hidden_size=16, num_heads=2, key_dim=8, value_dim=8, gate_cap=5.0, eps=1e-6)
    for change in (dict(key_dim=600), dict(gate_cap=0.0), dict(names={"z": "z"})):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("mlstm", {**mlstm, **change}), prefix="m")
    lightning = dict(hidden_size=16, num_heads=2, key_dim=8, value_dim=8, decay=(0.5, 0.6), eps=1e-6)
    for change in (dict(key_dim=600), dict(decay=(0.5,)), dict(names={"z": "z"})):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("lightning_attention", {**lightning, **change}), prefix="m")
    with pytest.raises(ValueError, match="shared"):
        RoutedExperts("f", 16, 4, 2, 8, shared_gate=True)
    with pytest.raises(ValueError, match="activation"):
        ActivatedFF("f", 16, 8, activation="cubed_relu")


def test_the_input_rows_of_an_mlstm_are_padded_with_nothing():
    part = build_part("mixer", PartSpec("mlstm", {"hidden_size": 16, "num_heads": 3, "key_dim": 8, "value_dim": 12, "gate_cap": 5.0,
                                                  "eps": 1e-6, "suffix": ""}), prefix="m")
    assert sum(part.splits) == 126 and part.row_width == 128
    part.load(lambda name: torch.ones({s.name: s.shape for s in part.weight_specs()}[name]), Runtime(torch.float32, torch.device("cpu")))
    assert part.inputs.weight.shape == (128, 16) and not part.inputs.weight[126:].any() and part.inputs.weight[:126].all()


def test_a_stream_hands_out_its_rows_until_something_is_added():
    h = torch.randn(3, 8)
    stream = ResidualStream(h)
    assert stream.rows(torch.float32) is h
    first = stream.rows(torch.bfloat16)
    assert first is stream.rows(torch.bfloat16) and torch.equal(first, h.to(torch.bfloat16))
    left = torch.zeros(3, 8, dtype=torch.bfloat16)
    stream.rewritten(left)
    assert stream.rows(torch.bfloat16) is left
    stream.rewritten()
    assert torch.equal(stream.rows(torch.bfloat16), h.to(torch.bfloat16))


def test_plain_memory_against_the_sum_over_all_tokens():
    """The plain cell's memory, unrolled: every earlier token weighed by its input gate and the forget gates since, the size
    bounded by one (times the constant's share, which the maxima set)."""
    gen = torch.Generator().manual_seed(1)
    T, H, D, P = 9, 2, 3, 4
    q, k, v = (torch.randn(T, H, n, generator=gen, dtype=torch.float64) for n in (D, D, P))
    i, f = torch.randn(T, H, generator=gen, dtype=torch.float64) * 3, plain.log_sigmoid(torch.randn(T, H, generator=gen, dtype=torch.float64))
    got = plain.mlstm_cell(q, k, v, i, f)
    m = torch.zeros(H, dtype=torch.float64)
    for t in range(T):
        m = torch.maximum(f[t] + m, i[t])
        top, size = torch.zeros(H, P, dtype=torch.float64), torch.zeros(H, dtype=torch.float64)
        for j in range(t + 1):
            weight = torch.exp(i[j] + f[j + 1:t + 1].sum(dim=0)) * (k[j] * q[t]).sum(dim=1)
            top, size = top + weight[:, None] * v[j], size + weight
        want = top / (torch.clamp(size.abs(), min=1.0) + 1e-6 * torch.exp(m))[:, None]
        torch.testing.assert_close(got[t], want, rtol=1e-9, atol=1e-12)
