"""Each mechanism of the Tomopel decoder alone: the part with its kernels and the engine's cache manager against the
plain function written from the equations."""

import math

import pytest
import torch

from gizilorn_helpers import PartEngine, load_part, random_weights, rounded
from plain import tomopel_plain as plain
from test_gpu_gizilorn_parts import check
from somi_inference_amd.kernels import attention as attention_kernels
from somi_inference_amd.kernels import ops
from somi_inference_amd.parts import PartSpec, ResidualStream, Runtime, build_part

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
DEV = torch.device("cuda:0")
EPS = 1e-5


# ------------------------------------------------------------------------------------------ attention
def attention_part(heads, kv, dim, vdim, scale, bias_max, buckets, temp=None, hidden=48):
    spec = PartSpec("biased_attention", {"hidden_size": hidden, "num_heads": heads, "num_kv_heads": kv, "dim": dim,
                                         "value_dim": vdim, "scale": scale, "eps": EPS, "bias_max": bias_max,
                                         "buckets": buckets, "temperature": temp, "suffix": ""})
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "bias_max": bias_max}
    if temp:
        m["q_temp"] = {"coef": temp[0], "every": temp[1]}
    return build_part("mixer", spec, prefix="m"), m


SIZES = [  # heads, kv, dim, vdim, scale, bias_max, buckets, temperature, page
    (4, 2, 16, 16, 0.5, 40, 8, (0.6, 7), 8),            # kept in 32 channels
    (6, 2, 24, 40, 0.4, 90, 10, (1.2, 3), 4),           # three heads a key/value head, 48 kept channels
    (4, 4, 64, 64, 0.25, 128, 16, None, 16),            # the 32 x 32 tile kernel
    (3, 1, 128, 96, 0.15, 60, 12, (0.5, 50), 16),       # the same with values padded to the keys' size
    (20, 1, 48, 48, 0.3, 25, 6, (0.4, 11), 16),         # more heads a key/value head than a block of query slots has
    (2, 1, 33, 20, 0.4, 300, 7, None, 16),              # a bias that reaches past the whole sequence
    (2, 2, 144, 16, 0.15, 40, 8, (0.3, 20), 8),         # heads the matrix-core kernels with a bias are not built for
    (4, 2, 32, 32, 0.4, 40, 8, (0.3, 20), 12),          # pages of no power of two
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv,dim,vdim,scale,bias_max,buckets,temp,page", SIZES)
def test_attention_whole_cut_and_side_by_side(dtype, heads, kv, dim, vdim, scale, bias_max, buckets, temp, page):
    part, m = attention_part(heads, kv, dim, vdim, scale, bias_max, buckets, temp)
    w = random_weights(part, heads * dim, scale={"rel": 1.5, "g": 0.3})
    load_part(part, w, dtype, DEV)
    gen = torch.Generator().manual_seed(dim)
    x = rounded(torch.randn(170, 48, generator=gen), dtype)
    other = rounded(torch.randn(37, 48, generator=gen), dtype)
    want, want_other = plain.attention(x, w, "m.", m, EPS), plain.attention(other, w, "m.", m, EPS)
    engine = PartEngine([part], dtype, DEV, page, num_blocks=64)
    whole = engine.run_cut("a", x, [170])[0]
    check(whole, want, dtype)
    for sizes in ([1], [2], [7, 1, 1, 30], [64, 3]):
        cut = engine.run_cut("a", x, sizes)[0]
        check(cut, want, dtype)
        if dtype == torch.float32:
            torch.testing.assert_close(cut, whole, rtol=2e-5, atol=2e-5)
    # two requests in the same steps, in pages that others have just given back
    got_a, got_b, at_a, at_b = [], [], 0, 0
    while at_a < 170 or at_b < 37:
        portions = []
        if at_a < 170:
            portions.append(("a", x[at_a:at_a + 13]))
        if at_b < 37:
            portions.append(("b", other[at_b:at_b + (1 if at_b > 5 else 3)]))
        outs = engine.run(portions)[0]
        if at_a < 170:
            got_a.append(outs[0])
            at_a += 13
        if at_b < 37:
            got_b.append(outs[-1])
            at_b += portions[-1][1].shape[0]
    check(torch.cat(got_a), want, dtype)
    check(torch.cat(got_b), want_other, dtype)
    engine.cache.free("a")
    engine.cache.free("b")
    engine.cache.check_invariants()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,page", [(32, 8), (64, 16), (128, 16)])
def test_one_far_key_among_hundreds(dtype, dim, page):
    """The query of one token matches the key of one far token exactly; every other score is small.  It is found in a
    prompt, in a prompt's last portion and as a single token, at page borders and in the middle of pages."""
    part, m = attention_part(2, 1, dim, dim, 12.0 / dim, 50, 8, hidden=64)
    w = random_weights(part, dim, scale={"rel": 0.2, "g": 0.3})
    # keys read the first half of a row, queries the second half with the same matrix
    half = rounded(torch.randn(dim, 32, generator=torch.Generator().manual_seed(dim)) * 0.3)
    w["m.k"] = torch.cat([half, torch.zeros(dim, 32)], dim=1)
    w["m.q"] = torch.cat([torch.zeros(dim, 32), half], dim=1).repeat(2, 1)
    w["m.q.norm"], w["m.k.norm"] = torch.ones(dim), torch.ones(dim)
    load_part(part, w, dtype, DEV)
    engine = PartEngine([part], dtype, DEV, page, num_blocks=64)
    length = 420
    for far in (0, 1, page - 1, page, 5 * page + 3, 255, 256):
        x = rounded(torch.randn(length, 64, generator=torch.Generator().manual_seed(far)), dtype)
        x[length - 1, 32:] = x[far, :32]
        want = plain.attention(x, w, "m.", m, EPS)
        without = plain.attention(torch.cat([x[:far], -x[far:far + 1], x[far + 1:]]), w, "m.", m, EPS)
        assert float((want[-1] - without[-1]).norm()) > 0.3 * float(want[-1].norm())       # the key matters
        for sizes in ([length], [400, 20], [length - 1, 1], [length - 9, 9]):
            check(engine.run_cut("a", x, sizes)[0], want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,buckets,bias_max", [(32, 8, 40), (64, 16, 128), (128, 6, 200)])
def test_the_edges_of_every_distance_bucket(dtype, dim, buckets, bias_max):
    """A table whose one row lifts its keys above all others: attention is spread over that bucket's distances alone, so a
    bucket that begins or ends one distance off shows.  In prompts and in single tokens."""
    part, m = attention_part(2, 2, dim, dim, 0.02, bias_max, buckets)
    engine = PartEngine([part], dtype, DEV, 16, num_blocks=64)
    length = bias_max + 60
    x = rounded(torch.randn(length, 48, generator=torch.Generator().manual_seed(3)), dtype)
    for bucket in range(buckets):
        w = random_weights(part, 7, scale={"rel": 0.0, "g": 0.3})
        w["m.rel"] = torch.zeros(buckets, 2)
        w["m.rel"][bucket] = torch.tensor([24.0, 12.0])
        load_part(part, w, dtype, DEV)
        want = plain.attention(x, w, "m.", m, EPS)
        check(engine.run_cut("a", x, [length])[0], want, dtype)
        check(engine.run_cut("a", x, [length - 40] + [1] * 40)[0], want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_temperature_steps_at_multiples_of_its_period(dtype):
    """A large coefficient and a short period: a step one position early or late changes every score by a large share."""
    part, m = attention_part(2, 1, 32, 32, 0.1, 20, 8, temp=(3.0, 5))
    w = random_weights(part, 5, scale={"rel": 0.3, "g": 0.3})
    load_part(part, w, dtype, DEV)
    x = rounded(torch.randn(64, 48, generator=torch.Generator().manual_seed(8)), dtype)
    want = plain.attention(x, w, "m.", m, EPS)
    shifted = plain.attention(x, w, "m.", {**m, "q_temp": {"coef": 3.0, "every": 6}}, EPS)
    assert float((want - shifted).pow(2).mean().sqrt()) > 0.05 * float(want.pow(2).mean().sqrt())
    engine = PartEngine([part], dtype, DEV, 8)
    for sizes in ([64], [1], [3, 11]):
        check(engine.run_cut("a", x, sizes)[0], want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_with_its_keys_dealt_out_to_workgroups(dtype):
    """Decoding past a thousand keys: the keys of a token are split, only the split with the nearest keys meets the bias."""
    part, m = attention_part(4, 2, 64, 64, 0.3, 200, 12, temp=(0.5, 300))
    w = random_weights(part, 9, scale={"rel": 2.0, "g": 0.3})
    load_part(part, w, dtype, DEV)
    x = rounded(torch.randn(1300, 48, generator=torch.Generator().manual_seed(9)), dtype)
    want = plain.attention(x, w, "m.", m, EPS)
    engine = PartEngine([part], dtype, DEV, 16, num_blocks=100)
    check(engine.run_cut("a", x, [1100] + [1] * 200)[0], want, dtype)


@pytest.mark.parametrize("gate,norm,vnorm,bias", [(False, True, True, True), (True, False, True, True), (True, True, False, True), (True, True, True, False)])
def test_each_mechanism_of_the_attention_can_be_left_out(gate, norm, vnorm, bias):
    spec = PartSpec("biased_attention", {"hidden_size": 48, "num_heads": 4, "num_kv_heads": 2, "dim": 16, "value_dim": 24,
                                         "scale": 0.3, "eps": EPS, "bias_max": 30 if bias else None, "buckets": 8 if bias else None,
                                         "qk_norm": norm, "value_norm": vnorm, "gate": gate, "suffix": ""})
    part = build_part("mixer", spec, prefix="m")
    w = random_weights(part, 4, scale={"rel": 1.0})
    load_part(part, w, torch.float32, DEV)
    x = torch.randn(50, 48, generator=torch.Generator().manual_seed(4))
    got = PartEngine([part], torch.float32, DEV, 8).run_cut("a", x, [20, 1, 29])[0]
    # the plain function, mechanism by mechanism
    q, k, v = ((x @ w[f"m.{n}"].T).view(50, -1, d) for n, d in (("q", 16), ("k", 16), ("v", 24)))
    if norm:
        q, k = plain.rms(q, EPS) * w["m.q.norm"], plain.rms(k, EPS) * w["m.k.norm"]
    if vnorm:
        v = plain.rms(v, EPS)
    s = torch.einsum("ihd,jhd->hij", q, k.repeat_interleave(2, dim=1)) * 0.3
    if bias:
        s = s + plain.distance_bias(w["m.rel"], 50, 30)
    s = s.masked_fill(torch.ones(50, 50).triu(1).bool(), -math.inf)
    o = torch.einsum("hij,jhd->ihd", torch.softmax(s, dim=-1), v.repeat_interleave(2, dim=1))
    if gate:
        o = o * torch.sigmoid(x @ w["m.g"].T)[:, :, None]
    check(got, o.reshape(50, -1) @ w["m.o"].T, torch.float32)


def paged(n, nkv, dim, page, gen):
    """A request's keys and values in pages handed out in a shuffled order."""
    pages = (n + page - 1) // page
    order = torch.randperm(pages + 3, generator=gen)[:pages]
    k, v = torch.randn(n, nkv, dim, generator=gen), torch.randn(n, nkv, dim, generator=gen)
    kc, vc = torch.zeros(pages + 3, nkv, page, dim), torch.zeros(pages + 3, nkv, dim, page)
    for j in range(n):
        kc[order[j // page], :, j % page] = k[j]
        vc[order[j // page], :, :, j % page] = v[j]
    return (kc.to(torch.bfloat16).to(DEV), vc.to(torch.bfloat16).to(DEV), order.to(torch.int32).view(1, -1).to(DEV))


@pytest.mark.parametrize("dim,shape", [(64, 4), (64, 5), (128, 4), (128, 5), (64, 1), (64, 2), (128, 3), (96, 1), (48, 2), (80, 3)])
@pytest.mark.parametrize("length", [1, 90, 157, 11000])
def test_every_launch_shape_of_the_prompt_kernels_with_a_bias(dim, shape, length):
    """Against the plain kernel; a table of 11,000 distances does not fit LDS and is read where it lies."""
    gen = torch.Generator().manual_seed(dim + shape)
    n, nq, nkv = 330, 4, 2
    kc, vc, table = paged(n, nkv, dim, 16, gen)
    q = (torch.randn(n, nq * dim, generator=gen)).to(torch.bfloat16).to(DEV)
    bias = torch.randn(nq, length, generator=gen) * 2
    bias[:, -1] = 0.0
    bias = bias.to(DEV)
    start, first = torch.tensor([0, n], dtype=torch.int32, device=DEV), torch.zeros(1, dtype=torch.int32, device=DEV)
    positions = torch.arange(n, dtype=torch.int32, device=DEV)
    entry = torch.zeros(n, dtype=torch.int32, device=DEV)
    scale = dim ** -0.5
    want = ops.paged_attention_plain(q, q.shape[1], kc, vc, table, entry, positions, nq, 0, scale, bias)
    out = torch.empty_like(want)
    ops.attention_prefill(q, q.shape[1], kc, vc, table, start, first, n, nq, 0, scale, out, max_context=n, shape=shape, bias=bias)
    check(out, want, torch.bfloat16)
    for split_len, splits in ((384, 1), (64, 6)):
        ops.attention_decode(q, q.shape[1], kc, vc, table, entry, positions, nq, 0, scale, split_len, splits, out, bias=bias)
        check(out, want, torch.bfloat16)


@pytest.mark.parametrize("dim", [32, 64, 128])
@pytest.mark.parametrize("length", [2, 9, 21, 40])
def test_a_split_that_ends_just_beyond_the_bias_reads_no_leftover_of_another_launch(dim, length):
    """A split's last 32-key tile reaches past its keys and may come near enough for the bias though none of its keys
    does.  Before every launch another one, whose table is not a number anywhere, leaves its table in LDS."""
    gen = torch.Generator().manual_seed(dim + length)
    n, nq, nkv = 260, 4, 2
    kc, vc, table = paged(n, nkv, dim, 8, gen)
    q = torch.randn(n, nq * dim, generator=gen).to(torch.bfloat16).to(DEV)
    bias = torch.randn(nq, length, generator=gen) * 3
    bias[:, -1] = 0.0
    bias = bias.to(DEV)
    poison = torch.full((nq, 600), float("nan"), device=DEV)
    positions, entry = torch.arange(n, dtype=torch.int32, device=DEV), torch.zeros(n, dtype=torch.int32, device=DEV)
    want = ops.paged_attention_plain(q, q.shape[1], kc, vc, table, entry, positions, nq, 0, 0.2, bias)
    for split_len, splits in ((64, 5), (272, 1), (144, 2), (96, 3)):
        out, waste = torch.empty_like(want), torch.empty_like(want)
        ops.attention_decode(q, q.shape[1], kc, vc, table, entry, positions, nq, 0, 0.2, split_len, splits, waste, bias=poison)
        ops.attention_decode(q, q.shape[1], kc, vc, table, entry, positions, nq, 0, 0.2, split_len, splits, out, bias=bias)
        check(out, want, torch.bfloat16)


def test_sizes_without_a_matrix_core_kernel_for_the_bias_are_refused_by_it():
    gen = torch.Generator().manual_seed(1)
    kc, vc, table = paged(20, 1, 144, 8, gen)
    q = torch.randn(20, 144, generator=gen).to(torch.bfloat16).to(DEV)
    bias = torch.zeros(1, 5, device=DEV)
    assert not attention_kernels.forms_supported(kc, table)
    entry, positions = torch.zeros(20, dtype=torch.int32, device=DEV), torch.arange(20, dtype=torch.int32, device=DEV)
    with pytest.raises(ops.KernelError, match="distance bias"):
        ops.attention_decode(q, 144, kc, vc, table, entry, positions, 1, 0, 0.1, 64, 1, torch.empty_like(q), bias=bias)
    with pytest.raises(ops.KernelError, match="distance bias"):
        ops.attention_decode(q, 144, kc, vc, table, entry, positions, 1, 0, 0.1, 64, 1, torch.empty_like(q), bias=bias[:, 0])


# ------------------------------------------------------------------------------------------ Mamba-2
def mamba_part(heads, vdim, state, groups, taps, norm_groups, hidden=48):
    spec = PartSpec("mamba2", {"hidden_size": hidden, "num_heads": heads, "num_groups": groups, "state_dim": state,
                               "value_dim": vdim, "taps": taps, "norm_groups": norm_groups, "eps": EPS, "suffix": ""})
    return (build_part("mixer", spec, prefix="m"),
            {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": taps, "norm_groups": norm_groups})


MAMBA = [  # heads, vdim, state, groups, taps, normed parts
    (4, 16, 16, 2, 4, 2), (3, 10, 5, 1, 1, 1), (2, 24, 33, 2, 2, 3), (6, 7, 64, 3, 3, 6), (2, 40, 130, 1, 4, 1),
    (1, 66, 31, 1, 9, 2), (4, 8, 200, 2, 5, 4), (2, 5, 300, 1, 4, 1), (2, 64, 128, 1, 4, 1), (3, 20, 48, 3, 4, 2),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", MAMBA)
def test_mamba2_whole_cut_and_side_by_side(dtype, sizes):
    part, m = mamba_part(*sizes)
    w = random_weights(part, sum(sizes), scale={"in": 0.2})
    load_part(part, w, dtype, DEV)
    gen = torch.Generator().manual_seed(sum(sizes))
    x = rounded(torch.randn(150, 48, generator=gen), dtype)
    other = rounded(torch.randn(41, 48, generator=gen), dtype)
    want, want_other = plain.mamba2(x, w, "m.", m, EPS), plain.mamba2(other, w, "m.", m, EPS)
    engine = PartEngine([part], dtype, DEV, 8, num_blocks=64)
    whole = engine.run_cut("a", x, [150])[0]
    check(whole, want, dtype)
    for cuts in ([1], [2], [7, 1, 1, 30], [64, 3]):
        cut = engine.run_cut("a", x, cuts)[0]
        check(cut, want, dtype)
        if dtype == torch.float32:
            torch.testing.assert_close(cut, whole, rtol=2e-5, atol=2e-5)
    got_a, got_b, at = [], [], 0
    while at < 150:
        portions = [("a", x[at:at + 11])]
        b = other[at // 11 * 3:at // 11 * 3 + (3 if at % 22 else 1) * (at // 11 * 3 < 41)]
        if at // 11 < 13 and at // 11 * 3 < 41:
            portions.append(("b", other[at // 11 * 3:at // 11 * 3 + 3]))
        outs = engine.run(portions)[0]
        got_a.append(outs[0])
        if len(portions) > 1:
            got_b.append(outs[1])
        at += 11
    check(torch.cat(got_a), want, dtype)
    done = torch.cat(got_b)
    check(done, want_other[:done.shape[0]], dtype)


def step_of(lengths):
    """What the recurrence reads of a step with entries of these lengths, in slots that are not in order."""
    from types import SimpleNamespace
    starts = [0]
    for n in lengths:
        starts.append(starts[-1] + n)
    slots = [(3 * i + 1) % (3 * len(lengths)) for i in range(len(lengths))]
    return SimpleNamespace(entry_start=torch.tensor(starts, dtype=torch.int32, device=DEV), max_entry_len=max(lengths),
                           state_slots=torch.tensor(slots, dtype=torch.int32, device=DEV)), starts, slots


@pytest.mark.parametrize("heads,p,n_state,groups", [(2, 64, 128, 1), (4, 16, 16, 2), (3, 12, 20, 3), (2, 100, 36, 1), (1, 132, 256, 1), (6, 8, 4, 2)])
@pytest.mark.parametrize("lengths", [[64], [65], [127, 1, 128], [3, 200, 63, 64, 1, 333]])
def test_the_recurrence_in_chunks_is_the_recurrence_token_by_token(heads, p, n_state, groups, lengths):
    """Both forms from the same states, against each other and against the plain function in float64; decays from almost
    one to almost zero stand side by side in a chunk."""
    gen = torch.Generator().manual_seed(heads * p + len(lengths))
    step, starts, slots = step_of(lengths)
    n, total = starts[-1], heads * p + 2 * groups * n_state
    xbc, rows = torch.randn(n, total, generator=gen), torch.randn(n, heads + 3, generator=gen) * 3
    bias, a_log, skip = (torch.randn(heads, generator=gen) * s for s in (2.0, 1.5, 1.0))
    state = torch.randn(3 * len(lengths), heads, p, n_state, generator=gen)
    assert ops.ssd_chunked(p, n_state)
    got = {}
    for chunked in (True, False):
        kept = state.to(DEV)
        y = ops.ssd(xbc.to(DEV), rows.to(DEV)[:, 3:], bias.to(DEV), a_log.to(DEV), skip.to(DEV), step, kept, groups, chunked=chunked)
        got[chunked] = (y.cpu(), kept.cpu())
    for e, length in enumerate(lengths):
        at = slice(starts[e], starts[e] + length)
        x, b, c = torch.split(xbc[at].double(), [heads * p, groups * n_state, groups * n_state], dim=1)
        dt = plain.softplus(rows[at, 3:].double() + bias.double())
        b, c = b.view(length, groups, -1).repeat_interleave(heads // groups, 1), c.view(length, groups, -1).repeat_interleave(heads // groups, 1)
        s, want = state[slots[e]].double(), []
        for t in range(length):
            s = torch.exp(-torch.exp(a_log.double()) * dt[t])[:, None, None] * s + (dt[t][:, None] * x[t].view(heads, p))[:, :, None] * b[t][:, None, :]
            want.append((s * c[t][:, None, :]).sum(-1) + skip.double()[:, None] * x[t].view(heads, p))
        want = torch.stack(want).view(length, -1).float()
        for chunked in (True, False):
            torch.testing.assert_close(got[chunked][0][at], want, rtol=1e-4, atol=2e-5 * float(want.abs().max()))
            torch.testing.assert_close(got[chunked][1][slots[e]], s.float(), rtol=1e-4, atol=2e-5 * float(s.abs().max()))
    idle = [i for i in range(3 * len(lengths)) if i not in slots]
    assert all(torch.equal(got[chunked][1][idle], state[idle]) for chunked in (True, False))


def test_which_sizes_the_chunked_recurrence_takes():
    assert not ops.ssd_chunked(10, 16) and not ops.ssd_chunked(16, 33) and not ops.ssd_chunked(16, 300)


def test_the_state_remembers_and_the_next_request_starts_from_zero():
    """A slow decay: an early token still weighs hundreds of tokens later; a slot used again starts from zeros."""
    part, m = mamba_part(2, 16, 24, 1, 3, 1)
    w = random_weights(part, 3, scale={"in": 0.3})
    w["m.A_log"], w["m.dt_bias"] = torch.full((2,), -6.0), torch.full((2,), -1.0)
    load_part(part, w, torch.float32, DEV)
    x = torch.randn(400, 48, generator=torch.Generator().manual_seed(5))
    want = plain.mamba2(x, w, "m.", m, EPS)
    forgot = plain.mamba2(torch.cat([x[:3] * 0, x[3:]]), w, "m.", m, EPS)
    assert float((want[-1] - forgot[-1]).norm()) > 0.005 * float(want[-1].norm())
    engine = PartEngine([part], torch.float32, DEV, 8, max_requests=1)
    for _ in range(2):                       # the second time in the same slot
        check(engine.run_cut("a", x, [300] + [1] * 100)[0], want, torch.float32)


def test_the_step_sizes_are_not_clamped():
    """softplus far out on both sides: dt of about 60 (everything forgotten) and of e^-20 (nothing written)."""
    part, m = mamba_part(2, 8, 8, 1, 2, 1)
    w = random_weights(part, 11, scale={"in": 0.2})
    w["m.dt_bias"] = torch.tensor([60.0, -20.0])
    load_part(part, w, torch.float32, DEV)
    x = torch.randn(40, 48, generator=torch.Generator().manual_seed(6))
    check(PartEngine([part], torch.float32, DEV, 8).run_cut("a", x, [40])[0], plain.mamba2(x, w, "m.", m, EPS), torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,groups", [(48, 1), (48, 6), (5000, 1), (9000, 3)])
def test_gate_before_the_grouped_norm(dtype, width, groups):
    gen = torch.Generator().manual_seed(width)
    y, rows, w = torch.randn(5, width, generator=gen), torch.randn(5, width + 7, generator=gen), torch.randn(width, generator=gen)
    y[:, :width // groups] *= 20                                    # parts of unlike sizes
    z = rows[:, 7:]
    out = torch.zeros(5, width + 3, dtype=dtype, device=DEV)
    ops.gated_group_norm(y.to(DEV), rows.to(DEV)[:, 7:], w.to(DEV), groups, EPS, 0.7, out[:, 3:])
    check(out[:, 3:], 0.7 * plain.grouped_rms(y * plain.silu(z), groups, EPS) * w, dtype)
    assert not bool(out[:, :3].any())


# ------------------------------------------------------------------------------------------ minGRU
def gru_part(width, hidden=48):
    return build_part("mixer", PartSpec("min_gru", {"hidden_size": hidden, "width": width, "suffix": ""}), prefix="m")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [7, 32, 40, 130])
def test_min_gru_whole_cut_and_side_by_side(dtype, width):
    part = gru_part(width)
    w = random_weights(part, width)
    load_part(part, w, dtype, DEV)
    gen = torch.Generator().manual_seed(width)
    x = rounded(torch.randn(330, 48, generator=gen), dtype)
    other = rounded(torch.randn(30, 48, generator=gen), dtype)
    want, want_other = plain.min_gru(x, w, "m."), plain.min_gru(other, w, "m.")
    engine = PartEngine([part], dtype, DEV, 8, num_blocks=64)
    whole = engine.run_cut("a", x, [330])[0]
    check(whole, want, dtype)
    for cuts in ([1], [2], [7, 1, 1, 30], [16, 17], [256, 257], [8, 9]):
        cut = engine.run_cut("a", x, cuts)[0]
        check(cut, want, dtype)
        if dtype == torch.float32:
            torch.testing.assert_close(cut, whole, rtol=2e-5, atol=2e-5)
    for size, small in ((11, [1] * 30), (33, [1, 8, 9, 1, 2, 1, 1, 1, 1, 5])):
        got_a, got_b, at = [], [], 0
        for i, few in enumerate(small):      # few tokens of one request beside portions of the other
            outs = engine.run([("a", x[size * i:size * i + size]), ("b", other[at:at + few])])[0]
            at += few
            got_a.append(outs[0])
            got_b.append(outs[1])
        check(torch.cat(got_a), want, dtype)
        check(torch.cat(got_b), want_other, dtype)
        for rid in ("a", "b"):
            engine.cache.free(rid)


def test_min_gru_gates_far_out_and_the_candidate_on_both_sides_of_zero():
    """z of almost 0 keeps the state of long ago, z of almost 1 replaces it; candidates of u >= 0 and u < 0."""
    part = gru_part(32)
    w = random_weights(part, 1)
    w["m.z.b"] = torch.linspace(-12.0, 12.0, 32)
    w["m.x.b"] = torch.linspace(4.0, -4.0, 32)
    load_part(part, w, torch.float32, DEV)
    x = torch.randn(600, 48, generator=torch.Generator().manual_seed(2))
    want = plain.min_gru(x, w, "m.")
    engine = PartEngine([part], torch.float32, DEV, 8, num_blocks=100, max_requests=1)
    for _ in range(2):                       # the second time in the same slot
        check(engine.run_cut("a", x, [500] + [1] * 100)[0], want, torch.float32)


# ------------------------------------------------------------------------------------------ side by side
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("left_scale,right_scale,vdim", [(0.4, 1.7, 12), (1.0, 1.0, 16), (-0.6, 0.25, 13)])
def test_two_mixers_through_shared_products_and_each_through_its_own(dtype, left_scale, right_scale, vdim):
    left = {"hidden_size": 48, "num_heads": 4, "num_kv_heads": 2, "dim": 16, "value_dim": 24, "scale": 0.4, "eps": EPS,
            "bias_max": 30, "buckets": 8, "temperature": (0.5, 9), "suffix": ""}
    right = {"hidden_size": 48, "num_heads": 2, "num_groups": 1, "state_dim": 16, "value_dim": vdim, "taps": 3, "norm_groups": 2,
             "eps": EPS, "suffix": ""}
    part = build_part("mixer", PartSpec("parallel", {
        "hidden_size": 48, "join": "scaled_sum", "left_scale": left_scale, "right_scale": right_scale,
        "left": PartSpec("biased_attention", left), "right": PartSpec("mamba2", right)}), prefix="m")
    assert part.stacked
    w = random_weights(part, 13, scale={"rel": 1.0})
    m = {"left_scale": left_scale, "right_scale": right_scale,
         "left": {"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 24, "scale": 0.4, "bias_max": 30, "q_temp": {"coef": 0.5, "every": 9}},
         "right": {"heads": 2, "vdim": vdim, "state": 16, "groups": 1, "conv": 3, "norm_groups": 2}}
    x = rounded(torch.randn(70, 48, generator=torch.Generator().manual_seed(14)), dtype)
    want = plain.parallel(x, w, "m.", m, EPS)
    for stacked in (True, False):
        part.stacked = stacked
        load_part(part, w, dtype, DEV)
        engine = PartEngine([part], dtype, DEV, 8)
        for sizes in ([70], [30, 1, 2, 17]):
            check(engine.run_cut("a", x, sizes)[0], want, dtype)


# ------------------------------------------------------------------------------------------ feed-forwards
def experts_part(experts, top, ff, shared, width=64):
    return build_part("feed_forward", PartSpec("routed_experts", {
        "hidden_size": width, "num_experts": experts, "top": top, "expert_size": ff, "shared_size": shared,
        "unit": "squared_relu", "correction": True, "suffix": ""}), prefix="f")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("experts,top,ff,shared,rows,width", [
    (8, 2, 40, 24, 1, 64), (8, 2, 40, None, 37, 64), (5, 5, 24, 56, 70, 64), (4, 1, 64, 8, 300, 64), (16, 3, 136, 32, 530, 96),
    (6, 2, 20, 12, 33, 76), (3, 2, 21, 7, 40, 50), (70, 4, 16, 16, 90, 64)])
def test_experts_without_a_gate(dtype, experts, top, ff, shared, rows, width):
    part = experts_part(experts, top, ff, shared, width)
    w = random_weights(part, experts + rows, scale={"router": 0.3, "correction": 0.3})
    load_part(part, w, dtype, DEV)
    x = rounded(torch.randn(rows, width, generator=torch.Generator().manual_seed(rows)), dtype)
    mlp = {"router": {"top": top}, "shared": {"ff": shared} if shared else None}
    margins = []
    want = plain.experts(x, w, "f.", mlp, margins)
    clear = margins[0] > 1e-5                                    # x is exact in both, so only float32 ties are left out
    assert float(clear.float().mean()) > 0.95
    got = part.forward(x.to(dtype).to(DEV))
    check(got[clear.to(DEV)], want[clear], dtype)


def test_the_correction_moves_the_choice_and_not_the_weights():
    """Corrections far below minus one and above one: choice scores are negative, the chosen experts are those with the
    largest correction, the weights come from the scores alone."""
    part = experts_part(6, 2, 16, None)
    w = random_weights(part, 2, scale={"router": 0.4})
    w["f.correction"] = torch.tensor([-9.0, -2.5, -7.0, -3.0, -30.0, -8.0])
    load_part(part, w, torch.float32, DEV)
    x = torch.randn(20, 64, generator=torch.Generator().manual_seed(1))
    chosen, weight = ops.moe_route(x.to(DEV), part.router, 2, 1, 1, "softmax", True, part.correction)
    assert sorted(set(chosen.cpu().flatten().tolist())) == [1, 3]
    want_chosen, want_weight, _ = plain.route(x, w, "f.", 2)
    assert torch.equal(chosen.cpu().long(), want_chosen)
    torch.testing.assert_close(weight.cpu(), want_weight, rtol=1e-5, atol=1e-6)
    check(part.forward(x.to(DEV)), plain.experts(x, w, "f.", {"router": {"top": 2}}), torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
def test_squared_relu_on_both_sides_of_zero(dtype):
    z = torch.tensor([[-3.0, -0.0, 0.0, 1e-3, 0.5, 2.0, 30.0]])
    check(ops.squared_relu(z.to(DEV), dtype), torch.relu(z) ** 2, dtype)


# ------------------------------------------------------------------------------------------ the layer
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("streams,mult", [(3, 0.35), (1, 2.0), (None, 0.35)])
def test_the_residual_multiplier_scales_what_a_sublayer_adds(dtype, streams, mult):
    norm = {"hidden_size": 64, "eps": EPS, "around_one": True}
    block = build_part("block", PartSpec("hyper_connections", {
        "mixer": PartSpec("min_gru", {"hidden_size": 64, "width": 40, "suffix": ""}),
        "feed_forward": PartSpec("swiglu", {"hidden_size": 64, "intermediate_size": 48, "suffix": "",
                                            "names": {"gate": "gate", "up": "up", "down": "down"}}),
        "mixer_norm": PartSpec("rmsnorm", {**norm, "tensor": "norm1"}), "ffn_norm": PartSpec("rmsnorm", {**norm, "tensor": "norm2"}),
        "streams": streams or 1, "connections": streams is not None, "residual_mult": mult,
        "names": {"mixer_norm": "", "ffn_norm": "", "mixer": "mix", "feed_forward": "mlp"}}), prefix="l")
    w = random_weights(block, 21, scale={"in": 0.4, "out": 0.6, "mix": 0.5, "norm1": 0.3, "norm2": 0.3, "gate": 0.15, "up": 0.15, "down": 0.15})
    load_part(block, w, dtype, DEV)
    gen = torch.Generator().manual_seed(22)
    x = torch.randn(30, 64, generator=gen)
    lanes = x[None].repeat(streams or 1, 1, 1)
    for sub in (1, 2):
        u = plain.read_streams(lanes, w, f"l.hc{sub}.") if streams else lanes[0]
        h = plain.norm_around_one(u, w[f"l.norm{sub}"], EPS)
        y = plain.min_gru(h, w, "l.mix.") if sub == 1 else plain.dense(h, w, "l.mlp.")
        lanes = plain.write_streams(lanes, y, w, f"l.hc{sub}.", mult) if streams else lanes + mult * y[None]

    class Layer:                             # what the harness runs as a mixer
        entry_split = None

        def cache_spec(self):
            return block.cache_spec()

        def forward(self, rows, step, cache):
            stream = ResidualStream(x.to(DEV))
            block.forward(stream, step, cache)
            return stream.settle()
    got = PartEngine([Layer()], dtype, DEV, 8).run_cut("a", x, [30])[0]
    check(got, lanes.sum(dim=0), dtype)
