"""The Tomopel configuration, its plan, its distance buckets and what the plan asks of the cache manager (no GPU)."""

import copy
import dataclasses
import math

import pytest
import torch

from plain import tomopel_plain as plain
from tomopel_helpers import TOMOPEL
from somi_inference_amd.config import ConfigError, TomopelConfig, config_from_dict
from somi_inference_amd.models import DecoderModel, collect_weight_specs, tomopel_plan
from somi_inference_amd.parts import CompositeSpec, FixedStateSpec, PagedKVSpec, ParallelMixers, PartSpec, RMSNorm, Runtime, build_part
from somi_inference_amd.parts.biased_attention import distance_buckets


def raw(name="A"):
    return TOMOPEL[name]["config"].to_dict()


@pytest.mark.parametrize("name", list(TOMOPEL))
def test_config_round_trip_and_registry(name):
    config = TOMOPEL[name]["config"]
    arch, again = config_from_dict(config.to_dict())
    assert arch.name == "Tomopel" and again == config and isinstance(again, TomopelConfig)


def test_keys_a_model_may_leave_out():
    data = raw("A")
    del data["streams"], data["residual_mult"], data["embedding"]
    left = data["layers"][0]["mixer"]["left"]
    del left["q_temp"], left["buckets"]
    del data["layers"][0]["mlp"]["shared"]
    config = TomopelConfig.from_dict(data)
    assert config.streams is None and config.residual_mult == 1.0 and config.embedding_scale == 1.0
    attention = config.layers[0].mixer.left
    assert attention.temp_coef is None and attention.buckets is None and config.layers[0].mlp.shared_ff is None
    assert config.layers[2].mlp is None


@pytest.mark.parametrize("change,word", [
    (lambda d: d["layers"][0]["mixer"].pop("left"), "left"),
    (lambda d: d["layers"][0]["mixer"]["left"].update(kv_heads=4), "kv_heads"),
    (lambda d: d["layers"][0]["mixer"]["left"].pop("bias_max"), "bias_max"),
    (lambda d: d["layers"][0]["mixer"]["left"].update(bias_max=5), "bias_max"),
    (lambda d: d["layers"][0]["mixer"]["left"].update(scale=0.0), "scale"),
    (lambda d: d["layers"][0]["mixer"]["left"]["q_temp"].update(every=0), "every"),
    (lambda d: d["layers"][0]["mixer"]["right"].update(groups=3), "groups"),
    (lambda d: d["layers"][0]["mixer"]["right"].update(norm_groups=5), "norm_groups"),
    (lambda d: d["layers"][1]["mixer"].pop("width"), "width"),
    (lambda d: d["layers"][1].update(type="recurrence"), "type"),
    (lambda d: d["layers"][0]["mlp"]["router"].update(top=7), "top"),
    (lambda d: d["layers"][0]["mlp"].update(kind="sparse"), "kind"),
    (lambda d: d.update(streams=0), "streams"),
])
def test_what_is_refused(change, word):
    data = copy.deepcopy(raw("A"))
    change(data)
    with pytest.raises(ConfigError, match=word):
        TomopelConfig.from_dict(data)


def test_tensor_names_and_shapes():
    specs = {s.name: s for s in collect_weight_specs(tomopel_plan(TOMOPEL["A"]["config"]))}
    assert specs["embed"].shape == (301, 96) and specs["head"].shape == (301, 96) and specs["final.norm"].shape == (96,)
    assert specs["l0.mix.left.q"].shape == (144, 96) and specs["l0.mix.left.k"].shape == (48, 96)
    assert specs["l0.mix.left.v"].shape == (32, 96) and specs["l0.mix.left.o"].shape == (96, 96)
    assert specs["l0.mix.left.g"].shape == (6, 96) and specs["l0.mix.left.rel"].shape == (10, 6)
    assert specs["l0.mix.left.q.norm"].shape == (24,) and specs["l0.mix.left.k.norm"].shape == (24,)
    assert specs["l0.mix.right.in"].shape == (2 * 48 + 2 * 2 * 20 + 4, 96) and specs["l0.mix.right.conv"].shape == (48 + 80, 4)
    assert specs["l0.mix.right.conv.b"].shape == (128,) and specs["l0.mix.right.norm"].shape == (48,)
    assert specs["l0.mix.right.A_log"].shape == (4,) and specs["l0.mix.right.o"].shape == (96, 48)
    assert specs["l1.mix.z"].shape == (72, 96) and specs["l1.mix.x.b"].shape == (72,) and specs["l1.mix.o"].shape == (96, 72)
    assert specs["l0.mlp.e5.up"].shape == (40, 96) and specs["l0.mlp.correction"].shape == (6,)
    assert specs["l0.mlp.shared.down"].shape == (96, 24) and "l0.mlp.e0.gate" not in specs and "l3.mlp.shared.up" not in specs
    assert specs["l1.mlp.gate"].shape == (64, 96) and "l2.mlp.up" not in specs and "l2.hc2.in" not in specs
    assert specs["l2.hc1.mix"].shape == (3, 3) and specs["l0.hc2.out"].shape == (3,)
    assert not any(name.endswith((".weight", ".bias")) for name in specs)
    assert not any(".hc" in s.name for s in collect_weight_specs(tomopel_plan(TOMOPEL["C"]["config"])))
    one_stream = {s.name: s for s in collect_weight_specs(tomopel_plan(TOMOPEL["B"]["config"]))}
    assert one_stream["l0.hc1.mix"].shape == (1, 1)


def test_what_the_checkpoint_says():
    """The rows of the bias tables, and, for one stream or none named, whether there are connection tensors."""
    config = TOMOPEL["B"]["config"]
    data = config.to_dict()
    del data["layers"][1]["mixer"]["left"]["buckets"]
    open_config = TomopelConfig.from_dict(data)
    shapes = {s.name: s.shape for s in collect_weight_specs(tomopel_plan(config))}
    assert open_config.layers[1].mixer.left.buckets is None and open_config.fitted_to(shapes) == config
    without = {name: shape for name, shape in shapes.items() if ".hc" not in name}
    assert config.fitted_to(without).streams is None
    none = TOMOPEL["C"]["config"]
    assert none.fitted_to({"l0.mix.left.rel": (7, 3)}) == none
    assert none.fitted_to({"l0.hc1.in": (2,), "l0.hc1.mix": (2, 2)}).streams == 2
    three = TOMOPEL["A"]["config"]
    assert three.fitted_to({}).streams == 3                      # three streams need their tensors: the loader says so
    with pytest.raises(ConfigError, match="bias_max"):           # a table with more rows than the farthest distance allows
        open_config.fitted_to({"l1.mix.left.rel": (400, 4)})


def test_what_a_layer_keeps():
    model = DecoderModel(tomopel_plan(TOMOPEL["A"]["config"]), Runtime(torch.float32, torch.device("cpu")))
    first, second, third, _ = model.cache_needs()
    assert isinstance(first, CompositeSpec) and isinstance(second, FixedStateSpec) and second.shape == (72,)
    kept = dict(first.parts)
    assert isinstance(kept["left"], PagedKVSpec) and kept["left"].num_kv_heads == 2 and kept["left"].head_dim == 32
    right = dict(kept["right"].parts)
    assert right["state"].shape == (4, 12, 20) and right["conv"].shape == (3, 128)
    assert right["state"].dtype == right["conv"].dtype == second.dtype == torch.float32
    assert dict(third.parts)["left"].head_dim == 48              # one size for keys of 16 and values of 40 channels
    assert model.entry_splits() == [8] and model.graph_safe()


@pytest.mark.parametrize("buckets,farthest", [(10, 60), (16, 128), (16, 240), (7, 19), (2, 5), (3, 2), (32, 128), (24, 190), (4, 300), (12, 4096)])
def test_distance_buckets(buckets, farthest):
    mine = distance_buckets(buckets, farthest)
    assert mine == [plain.bucket_of(n, buckets, farthest) for n in range(len(mine))]
    assert mine[-1] == buckets - 1 and (len(mine) == 1 or mine[-2] < buckets - 1) and mine == sorted(mine)
    assert all(plain.bucket_of(n, buckets, farthest) == buckets - 1 for n in (len(mine), farthest, 10 * farthest))
    half = buckets // 2
    for n, bucket in enumerate(mine):
        if n < half:
            assert bucket == n
            continue
        steps = math.log(n / half) / math.log(farthest / half) * (buckets - half)
        if abs(steps - round(steps)) > 1e-9:                      # away from an edge the logarithms say the same
            assert bucket == min(buckets - 1, half + math.floor(steps))


def test_a_distance_on_a_bucket_edge_is_in_the_farther_bucket():
    # 8 (128 / 8)^(2 / 8) = 16 and 8 (128 / 8)^(4 / 8) = 32 exactly
    mine = distance_buckets(16, 128)
    assert (mine[15], mine[16], mine[31], mine[32], mine[63], mine[64]) == (9, 10, 11, 12, 13, 14)


@pytest.mark.parametrize("buckets,farthest", [(1, 10), (8, 4), (8, 3)])
def test_buckets_that_make_no_sense_are_refused(buckets, farthest):
    with pytest.raises(ValueError):
        distance_buckets(buckets, farthest)


def test_a_norm_around_one_adds_one_to_the_stored_weight():
    part = build_part("norm", PartSpec("rmsnorm", {"hidden_size": 3, "eps": 1e-6, "tensor": "n", "around_one": True}), prefix="x")
    assert isinstance(part, RMSNorm) and part.weight_specs()[0].init.mean == 0.0
    part.load(lambda name: torch.tensor([0.5, -0.25, 0.0]), Runtime(torch.float32, torch.device("cpu")))
    assert part.weight.tolist() == [1.5, 0.75, 1.0]


def test_parallel_mixers_are_joined_in_one_of_two_ways():
    gru = PartSpec("min_gru", {"hidden_size": 8, "width": 8})
    with pytest.raises(ValueError, match="joined"):
        ParallelMixers("p", 8, gru, gru, join="product")
    with pytest.raises(ValueError, match="eps"):
        ParallelMixers("p", 8, gru, gru)
    summed = ParallelMixers("p", 8, gru, gru, join="scaled_sum")
    assert summed.stacked and not any(s.name.endswith(".out") for s in summed.weight_specs())
    hgrn = PartSpec("hgrn2", {"hidden_size": 8, "num_heads": 1, "key_dim": 8, "value_dim": 8, "eps": 1e-6})
    assert not ParallelMixers("p", 8, gru, hgrn, join="scaled_sum").stacked


def test_sizes_no_kernel_takes_are_refused_when_the_part_is_built():
    base = dict(hidden_size=16, num_heads=4, num_kv_heads=2, dim=16, value_dim=16, scale=0.2, eps=1e-6)
    for change in (dict(num_kv_heads=3), dict(value_dim=300), dict(scale=0.0)):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("biased_attention", {**base, **change}), prefix="m")
    right = dict(hidden_size=16, num_heads=4, num_groups=2, state_dim=8, value_dim=6, taps=4, norm_groups=2, eps=1e-6)
    for change in (dict(num_groups=3), dict(norm_groups=5), dict(taps=10), dict(taps=0)):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("mamba2", {**right, **change}), prefix="m")


def test_random_configurations_keep_their_sizes_through_the_plan():
    config = dataclasses.replace(TOMOPEL["A"]["config"], residual_mult=0.3)
    block = tomopel_plan(config).layers[0].block
    assert block.params["residual_mult"] == 0.3 and block.params["streams"] == 3 and block.params["connections"]
