"""Random small Tomopel configurations (layer orders, one to eight streams or none, heads of any size over any number of
key/value heads, value sizes unlike key sizes, tables of few and many buckets, bias reaches shorter and longer than the
sequences, temperatures or none, groups, normed parts and taps of the recurrence, minGRU widths, dense and routed
feed-forwards or none, widths that are no multiple of 8, page sizes) under random mixed traces with so few pages that they
are used again: the engine against the plain implementation and against itself on the whole prompt.  Pages, states and
the memory the engine allocates from hold values that are not numbers before it starts."""

import random

import pytest
import torch

from helpers import make_engine, mixed_trace, peak_pages, token_ids
from plain import tomopel_plain as plain
from test_gpu_tomopel_model import assert_close, close_rows
from tomopel_helpers import TOMOPEL, load_plain, mingru, parallel, write_tomopel
from somi_inference_amd.config import TomopelConfig, TomopelDense, TomopelExperts
from somi_inference_amd.engine import StepEntry

pytestmark = pytest.mark.gpu


def random_config(rng: random.Random) -> TomopelConfig:
    def mlp():
        kind = rng.random()
        if kind < 0.2:
            return None
        if kind < 0.5:
            return TomopelDense(rng.choice([8, 20, 36, 64, 96]))
        experts = rng.choice([1, 2, 3, 5, 8, 17])
        return TomopelExperts(experts, rng.randint(1, min(experts, 4)), rng.choice([8, 12, 24, 40]), rng.choice([None, 4, 16, 40]))

    layers = []
    for _ in range(rng.choice([1, 2, 3, 4])):
        if rng.random() < 0.35:
            layers.append(mingru(rng.choice([1, 16, 31, 48, 100]), mlp()))
            continue
        kv = rng.choice([1, 2, 3, 4])
        dim = rng.choice([8, 13, 16, 24, 32, 48, 64, 96, 128, 136])
        buckets = rng.choice([2, 3, 6, 8, 16, 31])
        groups = rng.choice([1, 2, 3])
        heads = groups * rng.choice([1, 2, 3])
        vdim = rng.choice([3, 8, 16, 20, 33])
        inner = heads * vdim
        left_vdim = dim if rng.random() < 0.4 else rng.choice([8, 10, 24, 40, 64])
        layers.append(parallel(
            kv * rng.choice([1, 2, 3, 4, 6]), kv, dim, left_vdim, rng.choice([0.5, 1.0, 2.0]) / dim ** 0.5,
            buckets // 2 + rng.choice([1, 2, 7, 25, 100, 500]), buckets, rng.choice([None, (0.5, 16), (1.0, 3), (0.2, 64)]),
            (heads, vdim, rng.choice([4, 16, 17, 32, 40, 64, 80]), groups, rng.choice([1, 2, 3, 4, 6]),
             rng.choice([n for n in (1, 2, 3, 4, 6) if inner % n == 0])),
            rng.choice([1.0, 0.5, 1.4]), rng.choice([1.0, 0.3, 0.9]), mlp()))
    return TomopelConfig(vocab=rng.choice([61, 97, 130, 256, 301]), width=rng.choice([40, 44, 64, 72, 100, 132]),
                         norm_eps=rng.choice([1e-6, 1e-5]), embedding_scale=rng.choice([1.0, 0.5, 3.0]),
                         residual_mult=rng.choice([1.0, 0.3, 0.7]), streams=rng.choice([None, 1, 2, 3, 4, 8]), layers=tuple(layers))


def leave_no_zeros(runner) -> None:
    """Whatever is read before it is written shows: the cache's tensors and freed device memory become not a number."""
    for cache in runner.cache.layer_caches:
        for leaf in cache.leaves():
            for tensor in list(leaf.tensors.values()) + ([leaf.state] if leaf.state is not None else []):
                tensor.fill_(float("nan"))
    held = [torch.full((size,), float("nan"), device="cuda:0") for size in (1 << 22, 1 << 18, 1 << 14, 1 << 10, 100) for _ in range(8)]
    del held


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(24))
def test_random_configuration_under_a_random_mixed_trace(seed, dtype, tmp_path):
    rng = random.Random(seed)
    config = random_config(rng)
    block_size = rng.choice([4, 8, 16, 32])
    TOMOPEL["random"] = dict(block_size=block_size, seed=rng.randrange(1000), config=config)
    try:
        folder = write_tomopel("random", str(tmp_path / "model"), peaky=rng.random() < 0.5)
    finally:
        del TOMOPEL["random"]
    weights, plain_config = load_plain(folder)
    lengths = {f"r{i}": rng.choice([1, 2, 3, 17, 33, 45, 64, 70, 100, 150]) for i in range(rng.randrange(3, 7))}
    requests = {rid: token_ids(config.vocab, n, rng.randrange(10000)) for rid, n in lengths.items()}
    sizes = tuple(rng.choice([1, 2, 3, 5, 7, 8, 9, 11, 16, 17, 31, 64, 65]) for _ in range(6))
    steps = mixed_trace(requests, seed=rng.randrange(1000), portion_sizes=sizes)
    pages = peak_pages(steps, block_size)
    runner, _ = make_engine(folder, dtype, block_size, pages, max_requests=4)
    leave_no_zeros(runner)
    rows = {rid: [] for rid in requests}
    for entries, ends in steps:
        batch = []
        for rid, start, count in entries:
            if not runner.cache.has(rid):
                runner.begin(rid)
            batch.append(StepEntry(rid, requests[rid][start:start + count], list(range(count))))
        logits = runner.step(batch).cpu()
        at = 0
        for rid, start, count in entries:
            rows[rid].append(logits[at:at + count])
            at += count
        for rid in ends:
            runner.end(rid)
        runner.cache.check_invariants()
    what = f"seed {seed} {dtype} {config.to_dict()} pages of {block_size}"
    for rid, tokens in requests.items():
        mixed = torch.cat(rows[rid])
        margins = []
        want = plain.forward(plain_config, weights, tokens, dtype=torch.float32, margins=margins)[0]
        close = close_rows(margins)
        assert_close(mixed, want, dtype, f"{what}: request {rid} of {lengths[rid]} in a mixed trace", close)
        runner.begin("whole")
        whole = runner.step([StepEntry("whole", tokens, list(range(len(tokens))))]).cpu()
        runner.end("whole")
        if dtype == "float32":
            torch.testing.assert_close(mixed, whole, atol=3e-5, rtol=3e-5, msg=lambda m: f"{what}: logits of {rid} depend on the cutting: {m}")
        else:
            assert_close(mixed, whole, dtype, f"{what}: request {rid} against its whole prompt", close)
    assert runner.cache.free_pages() == [g.pool.num_pages for g in runner.cache.groups]
