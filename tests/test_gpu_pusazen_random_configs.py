"""Random small Pusazen configurations (layer orders, heads of any size over any number of key/value heads, value sizes unlike
key sizes, chunks shorter and longer than pages, key tiles and sequences, partial and whole rotations, caps that bite and
caps that do not, decays from almost zero to one, gate caps, dense and routed feed-forwards or none, widths that are no
multiple of 8, page sizes) under random mixed traces with so few pages that they are used again: the engine against the plain
implementation and against itself on the whole prompt.  Pages, states and the memory the engine allocates from hold values
that are not numbers before it starts."""

import random

import pytest
import torch

from helpers import make_engine, mixed_trace, peak_pages, token_ids
from test_gpu_pusazen_model import assert_close, assert_same, reference
from pusazen_helpers import PUSAZEN, attention, lightning, load_plain, mlstm, write_pusazen
from somi_inference_amd.config import PusazenConfig, PusazenDense, PusazenExperts
from somi_inference_amd.engine import StepEntry

pytestmark = pytest.mark.gpu


def random_config(rng: random.Random) -> PusazenConfig:
    def mlp():
        kind = rng.random()
        if kind < 0.2:
            return None
        if kind < 0.5:
            return PusazenDense(rng.choice([8, 20, 36, 64, 96]))
        experts = rng.choice([1, 2, 3, 5, 8, 17])
        return PusazenExperts(experts, rng.randint(1, min(experts, 4)), rng.choice([8, 12, 24, 40]), rng.choice([None, 4, 16, 40]))

    layers = []
    for _ in range(rng.choice([1, 2, 3, 4])):
        kind = rng.random()
        heads, dim, vdim = rng.choice([1, 2, 3, 5]), rng.choice([4, 8, 13, 16, 24, 33, 48, 64, 100]), rng.choice([3, 8, 16, 20, 33, 64, 68])
        if kind < 0.35:
            layers.append(mlstm(heads, dim, vdim, rng.choice([3.0, 10.0, 15.0, 30.0]), mlp()))
        elif kind < 0.6:
            layers.append(lightning(dim, vdim, [rng.choice([0.1, 0.7, 0.95, 0.999, 1.0]) for _ in range(heads)], mlp()))
        else:
            kv = rng.choice([1, 2, 3, 4])
            dim = rng.choice([8, 13, 16, 24, 32, 48, 64, 96, 128, 136])
            vdim = dim if rng.random() < 0.4 else rng.choice([8, 10, 24, 40, 64])
            dims = rng.choice([2, 4, 8, dim // 2 * 2, dim // 4 * 2])
            layers.append(attention(kv * rng.choice([1, 2, 3, 4, 6]), kv, dim, vdim, rng.choice([0.5, 1.0, 2.0]) / dim ** 0.5,
                                    rng.choice([2.0, 15.0, 50.0]), rng.choice([50.0, 10000.0]), max(2, dims),
                                    rng.choice([1, 3, 7, 16, 31, 32, 50, 64, 100, 129, 1000]), mlp()))
    return PusazenConfig(vocab=rng.choice([61, 97, 130, 256, 301]), width=rng.choice([40, 44, 64, 72, 100, 132]),
                         norm_eps=rng.choice([1e-6, 1e-5]), alpha=rng.choice([1.0, 2.0, 3.3]), logit_scale=rng.choice([1.0, 0.5, 3.0]),
                         layers=tuple(layers))


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
    PUSAZEN["random"] = dict(block_size=block_size, seed=rng.randrange(1000), config=config)
    try:
        folder = write_pusazen("random", str(tmp_path / "model"), peaky=rng.random() < 0.5)
    finally:
        del PUSAZEN["random"]
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
        want, allow = reference(plain_config, weights, tokens)
        assert_close(mixed, want, dtype, f"{what}: request {rid} of {lengths[rid]} in a mixed trace", allow)
        runner.begin("whole")
        whole = runner.step([StepEntry("whole", tokens, list(range(len(tokens))))]).cpu()
        runner.end("whole")
        if dtype == "float32":
            assert_same(mixed, whole, f"{what}: logits of {rid} depend on the cutting", allow)
        else:
            assert_close(mixed, whole, dtype, f"{what}: request {rid} against its whole prompt", allow)
    assert runner.cache.free_pages() == [g.pool.num_pages for g in runner.cache.groups]
