"""Each mechanism of the Pusazen decoder alone: the part with its kernels and the engine's cache manager against the plain
function written from the equations."""

from types import SimpleNamespace

import pytest
import torch

from gizilorn_helpers import PartEngine, load_part, random_weights, rounded
from plain import pusazen_plain as plain
from test_gpu_gizilorn_parts import check
from somi_inference_amd.kernels import attention as attention_kernels
from somi_inference_amd.kernels import ops
from somi_inference_amd.parts import PartSpec, ResidualStream, build_part

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
DEV = torch.device("cuda:0")
EPS = 1e-5


def side_by_side(engine, x, other, size, few):
    """Portions of ``size`` tokens of one request beside portions of ``few`` (cycled) of another, in the same steps; both
    requests' rows, their pages and slots given back."""
    got, at, turn = ([], []), [0, 0], 0
    while at[0] < x.shape[0] or at[1] < other.shape[0]:
        portions = []
        for index, (rid, rows, count) in enumerate((("a", x, size), ("b", other, few[turn % len(few)]))):
            if at[index] < rows.shape[0]:
                portions.append((index, rid, rows[at[index]:at[index] + count]))
                at[index] += count
        for (index, _, _), out in zip(portions, engine.run([(rid, rows) for _, rid, rows in portions])[0]):
            got[index].append(out)
        turn += 1
    for rid in ("a", "b"):
        engine.cache.free(rid)
    engine.cache.check_invariants()
    return torch.cat(got[0]), torch.cat(got[1])


# ------------------------------------------------------------------------------------------ attention
def attention_part(heads, kv, dim, vdim, scale, cap, base, dims, chunk, hidden=48):
    position = PartSpec("rotary", {"head_dim": dim, "theta": base, "rotary_dim": dims, "double": True}) if dims else PartSpec("none", {})
    spec = PartSpec("gqa_attention", {
        "hidden_size": hidden, "num_heads": heads, "num_kv_heads": kv, "head_dim": dim, "value_dim": vdim, "position": position,
        "qkv_bias": False, "scale": scale, "qk_norm": "projection", "norm_eps": EPS, "chunk": chunk, "softcap": cap, "sink": True,
        "suffix": "", "names": {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm"}})
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "softcap": cap,
         "rot": {"base": base, "dims": dims}, "mask": {"size": chunk}}
    return build_part("mixer", spec, prefix="m"), m


SIZES = [  # heads, kv, dim, vdim, scale, cap, base, dims, chunk, page
    (4, 2, 16, 16, 0.5, 20.0, 100.0, 8, 50, 8),             # kept in 32 channels
    (6, 2, 24, 40, 0.4, 3.0, 10000.0, 24, 33, 4),           # three heads a key/value head, 48 kept channels
    (4, 4, 64, 64, 0.25, 50.0, 1000.0, 16, 100, 16),        # the 32 x 32 tile kernel
    (3, 1, 128, 96, 0.15, 5.0, 500.0, 128, 64, 16),         # the same with values padded to the keys' size, chunks of whole pages
    (20, 1, 48, 48, 0.3, 30.0, 50.0, 2, 7, 16),             # more heads a key/value head than a block of query slots has
    (2, 1, 33, 20, 0.4, 8.0, 2000.0, 32, 300, 16),          # one chunk holds the whole sequence
    (2, 2, 144, 16, 0.15, 9.0, 10000.0, 96, 40, 8),         # heads the matrix-core kernels with such scores are not built for
    (4, 2, 32, 32, 0.4, 15.0, 10000.0, 32, 41, 12),         # pages of no power of two
    (2, 1, 64, 64, 0.4, 15.0, 10000.0, 64, 1, 16),          # a token sees itself and the sink alone
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv,dim,vdim,scale,cap,base,dims,chunk,page", SIZES)
def test_attention_whole_cut_and_side_by_side(dtype, heads, kv, dim, vdim, scale, cap, base, dims, chunk, page):
    part, m = attention_part(heads, kv, dim, vdim, scale, cap, base, dims, chunk)
    w = random_weights(part, heads * dim, scale={"sink": 2.0})
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
    got, got_other = side_by_side(engine, x, other, 13, [3, 3, 1])
    check(got, want, dtype)
    check(got_other, want_other, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim,page,chunk", [(32, 8, 150), (64, 16, 192), (64, 16, 131), (128, 16, 201), (48, 4, 96)])
def test_a_key_just_inside_and_just_outside_the_chunk(dtype, dim, page, chunk):
    """The query of one token matches one key; every other score is small.  The chunk's first key is found, the key before
    it is not, in a prompt, in a prompt's last portion and as a single token."""
    part, m = attention_part(2, 1, dim, dim, 9.0 / dim, 50.0, 10000.0, 2, chunk, hidden=64)
    w = random_weights(part, dim, scale={"sink": 1.0})
    # keys read the first half of a row, queries the second half with the same matrix
    half = rounded(torch.randn(dim, 32, generator=torch.Generator().manual_seed(dim)) * 0.3)
    w["m.k"] = torch.cat([half, torch.zeros(dim, 32)], dim=1)
    w["m.q"] = torch.cat([torch.zeros(dim, 32), half], dim=1).repeat(2, 1)
    w["m.q.norm"], w["m.k.norm"] = torch.ones(2 * dim), torch.ones(dim)
    load_part(part, w, dtype, DEV)
    engine = PartEngine([part], dtype, DEV, page, num_blocks=160)
    length = 2 * chunk + chunk // 2                           # the last token sees keys from 2 * chunk on
    for asked in (length - 1, 2 * chunk - 1):
        start = asked // chunk * chunk
        for far, seen in ((start, True), (start - 1, False), (start + 1, True), ((start // page + 1) * page, True), (0, False)):
            x = rounded(torch.randn(asked + 1, 64, generator=torch.Generator().manual_seed(far)), dtype)
            x[asked, 32:] = x[far, :32]
            want = plain.attention(x, w, "m.", m, EPS)
            without = plain.attention(torch.cat([x[:far], -x[far:far + 1], x[far + 1:]]), w, "m.", m, EPS)
            moved = float((want[-1] - without[-1]).norm()) / float(want[-1].norm())
            assert moved > 0.3 if seen else moved == 0.0
            for sizes in ([asked + 1], [asked - 19, 20], [asked, 1], [asked - 8, 9]):
                got = engine.run_cut("a", x, sizes)[0]
                check(got, want, dtype)
                check(got[-1:], want[-1:], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_every_token_around_a_chunks_edge_decoded(dtype):
    """Tokens decoded one by one across two edges; pages before a chunk are given back and used by another request."""
    part, m = attention_part(4, 2, 64, 64, 0.4, 20.0, 1000.0, 32, 72)
    w = random_weights(part, 3, scale={"sink": 1.0})
    load_part(part, w, dtype, DEV)
    x = rounded(torch.randn(220, 48, generator=torch.Generator().manual_seed(3)), dtype)
    want = plain.attention(x, w, "m.", m, EPS)
    engine = PartEngine([part], dtype, DEV, 16, num_blocks=16)
    check(engine.run_cut("a", x, [60] + [1] * 160)[0], want, dtype)
    held = []
    for at in range(0, 220, 10):
        engine.run([("b", x[at:at + 10])])
        held.append(16 - engine.cache.free_pages()[0])
    assert max(held) <= 6 and held[-1] == 1                   # position 220 lies in the chunk from 216, page 13
    engine.cache.free("b")


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_sink_counts_once_and_is_neither_scaled_nor_capped(dtype):
    """Sinks from far below every score to far above all: the output's size says how often and in which units they count."""
    part, m = attention_part(6, 3, 64, 64, 0.5, 2.0, 1000.0, 32, 600)
    w = random_weights(part, 5)
    w["m.sink"] = torch.tensor([-40.0, -1.0, 0.0, 3.0, 7.0, 30.0])
    load_part(part, w, dtype, DEV)
    x = rounded(torch.randn(700, 48, generator=torch.Generator().manual_seed(5)), dtype)
    want = plain.attention(x, w, "m.", m, EPS)
    doubled = plain.attention(x, {**w, "m.sink": w["m.sink"] + torch.log(torch.tensor(2.0))}, "m.", m, EPS)
    assert float((want - doubled).pow(2).mean().sqrt()) > 0.05 * float(want.pow(2).mean().sqrt())
    engine = PartEngine([part], dtype, DEV, 16, num_blocks=64)
    for sizes in ([700], [560] + [1] * 140, [599, 1, 100], [250, 9, 8]):
        got = engine.run_cut("a", x, sizes)[0]
        check(got, want, dtype)
        # the first tokens, whose denominators are mostly the sinks
        check(got[:4], want[:4], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_scores_far_beyond_the_cap(dtype):
    part, m = attention_part(2, 1, 32, 32, 6.0, 4.0, 1000.0, 16, 64)
    w = random_weights(part, 8, scale={"sink": 1.0})
    load_part(part, w, dtype, DEV)
    x = rounded(torch.randn(90, 48, generator=torch.Generator().manual_seed(8)), dtype)
    want = plain.attention(x, w, "m.", m, EPS)
    wider = plain.attention(x, w, "m.", {**m, "softcap": 5.0}, EPS)
    assert float((want - wider).pow(2).mean().sqrt()) > 0.05 * float(want.pow(2).mean().sqrt())
    engine = PartEngine([part], dtype, DEV, 8)
    for sizes in ([90], [1], [3, 11]):
        check(engine.run_cut("a", x, sizes)[0], want, dtype, loose=2.0)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_with_its_keys_dealt_out_to_workgroups(dtype):
    part, m = attention_part(4, 2, 64, 64, 0.3, 10.0, 10000.0, 64, 1150)
    w = random_weights(part, 9, scale={"sink": 3.0})
    load_part(part, w, dtype, DEV)
    x = rounded(torch.randn(1300, 48, generator=torch.Generator().manual_seed(9)), dtype)
    want = plain.attention(x.double(), {name: value.double() for name, value in w.items()}, "m.", m, EPS)
    engine = PartEngine([part], dtype, DEV, 16, num_blocks=100)
    # float32 angles of a thousand radians are off by some 1e-4
    check(engine.run_cut("a", x, [1100] + [1] * 200)[0], want, dtype, loose=6.0 if dtype == torch.float32 else 1.0)


def paged(n, nkv, dim, page, gen):
    """A request's keys and values in pages handed out in a shuffled order; one key in forty stands out."""
    pages = (n + page - 1) // page
    order = torch.randperm(pages + 3, generator=gen)[:pages]
    k, v = torch.randn(n, nkv, dim, generator=gen), torch.randn(n, nkv, dim, generator=gen)
    k[::40] *= 3
    kc, vc = torch.full((pages + 3, nkv, page, dim), float("nan")), torch.full((pages + 3, nkv, dim, page), float("nan"))
    for j in range(n):
        kc[order[j // page], :, j % page] = k[j]
        vc[order[j // page], :, :, j % page] = v[j]
    return (kc.to(torch.bfloat16).to(DEV), vc.to(torch.bfloat16).to(DEV), order.to(torch.int32).view(1, -1).to(DEV))


@pytest.mark.parametrize("dim,shape", [(64, 4), (64, 5), (128, 4), (128, 5), (64, 1), (64, 2), (128, 3), (96, 1), (48, 2), (80, 3)])
@pytest.mark.parametrize("cap,chunk,sink,window", [(6.0, 200, True, 0), (None, 77, False, 0), (3.0, None, False, 0), (None, None, True, 0),
                                                   (5.0, 128, True, 50)])
def test_every_launch_shape_of_the_prompt_kernels_with_such_scores(dim, shape, cap, chunk, sink, window):
    """Against the plain kernel, each of the three on its own and together, also beside a window."""
    gen = torch.Generator().manual_seed(dim + shape)
    n, nq, nkv = 330, 4, 2
    kc, vc, table = paged(n, nkv, dim, 16, gen)
    q = (torch.randn(n, nq * dim, generator=gen)).to(torch.bfloat16).to(DEV)
    score = ops.ScoreShape(cap, chunk, torch.randn(nq, generator=gen).mul(3).to(DEV) if sink else None)
    start, first = torch.tensor([0, n], dtype=torch.int32, device=DEV), torch.zeros(1, dtype=torch.int32, device=DEV)
    positions = torch.arange(n, dtype=torch.int32, device=DEV)
    entry = torch.zeros(n, dtype=torch.int32, device=DEV)
    scale = 1.5 * dim ** -0.5
    want = ops.paged_attention_plain(q, q.shape[1], kc, vc, table, entry, positions, nq, window, scale, None, score)
    out = torch.empty_like(want)
    ops.attention_prefill(q, q.shape[1], kc, vc, table, start, first, n, nq, window, scale, out, max_context=n, shape=shape, score=score)
    check(out, want, torch.bfloat16)
    for split_len, splits in ((384, 1), (64, 6)):
        ops.attention_decode(q, q.shape[1], kc, vc, table, entry, positions, nq, window, scale, split_len, splits, out, score=score)
        check(out, want, torch.bfloat16)


def test_sizes_without_a_matrix_core_kernel_for_such_scores_are_refused_by_it():
    gen = torch.Generator().manual_seed(1)
    kc, vc, table = paged(20, 1, 144, 8, gen)
    q = torch.randn(20, 144, generator=gen).to(torch.bfloat16).to(DEV)
    assert not attention_kernels.forms_supported(kc, table)
    entry, positions = torch.zeros(20, dtype=torch.int32, device=DEV), torch.arange(20, dtype=torch.int32, device=DEV)
    with pytest.raises(ops.KernelError, match="capped"):
        ops.attention_decode(q, 144, kc, vc, table, entry, positions, 1, 0, 0.1, 64, 1, torch.empty_like(q), score=ops.ScoreShape(chunk=5))
    with pytest.raises(ops.KernelError, match="sink"):
        ops.attention_decode(q, 144, kc, vc, table, entry, positions, 1, 0, 0.1, 64, 1, torch.empty_like(q),
                             score=ops.ScoreShape(sink=torch.zeros(2, device=DEV)))


@pytest.mark.parametrize("cap,chunk,sink", [(6.0, 40, True), (None, 24, False), (3.0, None, True)])
def test_such_scores_without_a_norm_over_the_projections(cap, chunk, sink):
    """The other path of the same part: heads rotated and stored without a norm."""
    spec = PartSpec("gqa_attention", {
        "hidden_size": 48, "num_heads": 4, "num_kv_heads": 2, "head_dim": 32, "qkv_bias": False, "scale": 0.3, "chunk": chunk,
        "softcap": cap, "sink": sink, "suffix": "", "names": {"q": "q", "k": "k", "v": "v", "o": "o"},
        "position": PartSpec("rotary", {"head_dim": 32, "theta": 1000.0})})
    part = build_part("mixer", spec, prefix="m")
    w = random_weights(part, 4, scale={"sink": 2.0})
    for dtype in DTYPES:
        load_part(part, w, dtype, DEV)
        x = rounded(torch.randn(90, 48, generator=torch.Generator().manual_seed(4)), dtype)
        q, k, v = ((x @ w[f"m.{n}"].T).view(90, -1, 32) for n in "qkv")
        s = torch.einsum("ihd,jhd->hij", plain.rotate(q, 1000.0, 32), plain.rotate(k, 1000.0, 32).repeat_interleave(2, dim=1)) * 0.3
        s = cap * torch.tanh(s / cap) if cap else s
        s = s.masked_fill(~plain.chunk_mask(90, chunk or 1000), float("-inf"))
        p = plain.sink_softmax(s, w["m.sink"]) if sink else torch.softmax(s, dim=-1)
        want = torch.einsum("hij,jhd->ihd", p, v.repeat_interleave(2, dim=1)).reshape(90, -1) @ w["m.o"].T
        for sizes in ([90], [40, 1, 9]):
            check(PartEngine([part], dtype, DEV, 8).run_cut("a", x, sizes)[0], want, dtype)


# ------------------------------------------------------------------------------------------ the recurrences
def mlstm_part(heads, dim, vdim, cap, hidden=48):
    spec = PartSpec("mlstm", {"hidden_size": hidden, "num_heads": heads, "key_dim": dim, "value_dim": vdim, "gate_cap": cap,
                              "eps": EPS, "suffix": ""})
    return build_part("mixer", spec, prefix="m"), {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def lightning_part(dim, vdim, decay, hidden=48):
    spec = PartSpec("lightning_attention", {"hidden_size": hidden, "num_heads": len(decay), "key_dim": dim, "value_dim": vdim,
                                            "decay": decay, "eps": EPS, "suffix": ""})
    return build_part("mixer", spec, prefix="m"), {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": decay}


RECURRENT = [
    ("mlstm", (4, 16, 16, 15.0)), ("mlstm", (3, 20, 12, 6.0)), ("mlstm", (1, 5, 7, 3.0)), ("mlstm", (2, 64, 64, 15.0)),
    ("mlstm", (2, 100, 130, 9.0)), ("mlstm", (1, 33, 20, 30.0)), ("mlstm", (2, 300, 8, 8.0)),
    ("lightning", (16, 16, [0.5, 0.9, 0.99, 1.0])), ("lightning", (20, 12, [0.01, 0.8, 0.999])), ("lightning", (5, 7, [0.9])),
    ("lightning", (64, 64, [0.97, 0.6])), ("lightning", (130, 100, [0.9, 0.99])), ("lightning", (33, 20, [0.95])),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,sizes", RECURRENT)
def test_recurrent_mixer_whole_cut_and_side_by_side(kind, sizes, dtype):
    part, m = (mlstm_part if kind == "mlstm" else lightning_part)(*sizes)
    w = random_weights(part, 7 * m["dim"] + m["vdim"], scale={"i": 0.4, "f": 0.4})
    load_part(part, w, dtype, DEV)
    gen = torch.Generator().manual_seed(m["dim"])
    x = rounded(torch.randn(170, 48, generator=gen), dtype)
    other = rounded(torch.randn(41, 48, generator=gen), dtype)
    want, want_other = (plain.MIXERS[kind](rows, w, "m.", m, EPS) for rows in (x, other))
    engine = PartEngine([part], dtype, DEV, 8, num_blocks=64)
    whole = engine.run_cut("a", x, [170])[0]
    check(whole, want, dtype)
    for cuts in ([1], [2], [7, 1, 1, 30], [64, 3], [65, 130]):
        cut = engine.run_cut("a", x, cuts)[0]
        check(cut, want, dtype)
        if dtype == torch.float32:
            torch.testing.assert_close(cut, whole, rtol=2e-5, atol=2e-5)
    for size, few in ((13, [3, 1]), (70, [1, 2, 30])):
        got, got_other = side_by_side(engine, x, other, size, few)
        check(got, want, dtype)
        check(got_other, want_other, dtype)


def step_of(lengths):
    """What the recurrence reads of a step with entries of these lengths, in slots that are not in order."""
    starts = [0]
    for n in lengths:
        starts.append(starts[-1] + n)
    slots = [(3 * i + 1) % (3 * len(lengths)) for i in range(len(lengths))]
    return SimpleNamespace(entry_start=torch.tensor(starts, dtype=torch.int32, device=DEV), max_entry_len=max(lengths),
                           state_slots=torch.tensor(slots, dtype=torch.int32, device=DEV)), starts, slots


@pytest.mark.parametrize("normaliser", [True, False])
@pytest.mark.parametrize("heads,p,d", [(2, 64, 128), (4, 16, 16), (3, 12, 20), (2, 100, 36), (1, 132, 256), (6, 8, 4)])
@pytest.mark.parametrize("lengths", [[64], [65], [127, 1, 128], [3, 200, 63, 64, 1, 333]])
def test_the_memory_in_chunks_is_the_memory_token_by_token(heads, p, d, lengths, normaliser):
    """Both forms from the same states, against each other and against the equations in float64; decays from almost one to
    almost zero stand side by side in a chunk."""
    gen = torch.Generator().manual_seed(heads * p + len(lengths))
    step, starts, slots = step_of(lengths)
    n = starts[-1]
    rows = torch.randn(n, heads * (2 * d + p) + 8, generator=gen)
    q, k, v = torch.split(rows[:, 4:-4], [heads * d, heads * d, heads * p], dim=1)
    keep = torch.rand(n, heads, generator=gen) ** torch.tensor([0.01, 4.0] * heads)[:heads] if normaliser else torch.rand(heads, generator=gen) ** 0.1
    write = torch.rand(n, heads, generator=gen) * 2 if normaliser else None
    state = torch.randn(3 * len(lengths), heads, p + int(normaliser), d, generator=gen)
    on_device = rows.to(DEV)
    views = torch.split(on_device[:, 4:-4], [heads * d, heads * d, heads * p], dim=1)
    got = {}
    for chunked in (True, False):
        kept = state.to(DEV)
        y, den = ops.ssd_memory(*views, step, kept, keep=keep.to(DEV), write=write.to(DEV) if normaliser else None, scale=0.3, chunked=chunked)
        got[chunked] = (y.cpu(), None if den is None else den.cpu(), kept.cpu())
    for e, length in enumerate(lengths):
        at = slice(starts[e], starts[e] + length)
        s, want = state[slots[e]].double(), []
        for t in range(starts[e], starts[e] + length):
            a = (keep[t] if normaliser else keep).double()[:, None, None]
            b = write[t].double()[:, None, None] if normaliser else 1.0
            x = v[t].double().view(heads, p)
            x = torch.cat([x, torch.ones(heads, 1, dtype=torch.float64)], dim=1) if normaliser else x
            s = a * s + b * x[:, :, None] * k[t].double().view(heads, 1, d)
            want.append(0.3 * (s * q[t].double().view(heads, 1, d)).sum(-1))
        want = torch.stack(want).float()
        for chunked in (True, False):
            y, den, kept = got[chunked]
            torch.testing.assert_close(y[at].view(length, heads, p), want[:, :, :p], rtol=1e-4, atol=2e-5 * float(want.abs().max()))
            if normaliser:
                torch.testing.assert_close(den[at], want[:, :, p], rtol=1e-4, atol=2e-5 * float(want.abs().max()))
            torch.testing.assert_close(kept[slots[e]], s.float(), rtol=1e-4, atol=2e-5 * float(s.abs().max()))
    idle = [i for i in range(3 * len(lengths)) if i not in slots]
    assert all(torch.equal(got[chunked][2][idle], state[idle]) for chunked in (True, False))


@pytest.mark.parametrize("lengths", [[1], [4, 1, 3], [5, 1], [1023, 1, 1025], [2500, 64]])
@pytest.mark.parametrize("heads", [3, 300])
def test_gates_and_running_maxima(lengths, heads):
    """Against the equations in float64, from maxima that earlier steps left: what is kept and written multiplies back to
    the same memory whatever the maxima were rounded to, and the maxima themselves agree."""
    gen = torch.Generator().manual_seed(sum(lengths))
    step, starts, slots = step_of(lengths)
    n, cap = starts[-1], 8.0
    rows = torch.randn(n, 2 * heads + 3, generator=gen) * 6
    rows[:, 3 + heads:] += torch.linspace(-9.0, 12.0, heads)              # forget gates from almost shut to almost open
    bias_i, bias_f = torch.randn(heads, generator=gen), torch.randn(heads, generator=gen)
    top = torch.randn(3 * len(lengths), heads, generator=gen) * 5
    kept = top.to(DEV)
    on_device = rows.to(DEV)
    keep, write, floor = (t.cpu().double() for t in ops.mlstm_gates(on_device[:, 3:3 + heads], on_device[:, 3 + heads:], bias_i.to(DEV),
                                                                    bias_f.to(DEV), cap, step, kept))
    i = cap * torch.tanh((rows[:, 3:3 + heads].double() + bias_i.double()) / cap)
    f = plain.log_sigmoid(cap * torch.tanh((rows[:, 3 + heads:].double() + bias_f.double()) / cap))
    for e, length in enumerate(lengths):
        m = top[slots[e]].double()
        for t in range(starts[e], starts[e] + length):
            before, m = m, torch.maximum(f[t] + m, i[t])
            torch.testing.assert_close(floor[t], torch.exp(-m), rtol=2e-5, atol=1e-9)
            torch.testing.assert_close(write[t], torch.exp(i[t] - m), rtol=2e-5, atol=1e-9)
            torch.testing.assert_close(keep[t], torch.exp(f[t] + before - m), rtol=2e-5, atol=1e-9)
        torch.testing.assert_close(kept[slots[e]].cpu().double(), m, rtol=1e-5, atol=1e-5)
    idle = [s for s in range(3 * len(lengths)) if s not in slots]
    assert torch.equal(kept[idle].cpu(), top[idle])


def test_the_running_maximum_starts_at_zero_and_the_normaliser_has_a_floor():
    """Input gates far below zero: the first tokens' outputs are small before their norm, and with an eps that is not small
    beside them the norm lets the floor show; a maximum that started at minus infinity would lift them."""
    part, m = mlstm_part(2, 16, 16, 15.0)
    w = random_weights(part, 2, scale={"i": 0.3, "f": 0.3})
    w["m.i.b"], w["m.f.b"] = torch.full((2,), -7.0), torch.full((2,), 4.0)
    load_part(part, w, torch.float32, DEV)
    x = torch.randn(120, 48, generator=torch.Generator().manual_seed(2))
    want = plain.mlstm(x, w, "m.", m, EPS)
    q, k, v = ((x @ w[f"m.{n}"].T).view(120, 2, 16) for n in "qkv")
    i, f = plain.mlstm_gates(x, w, "m.", 15.0)
    lifted = plain.mlstm_cell(q * 0.25, k, v, i + 50.0, f)                 # as if nothing bounded the size from below
    lifted = (plain.rms(lifted, EPS).reshape(120, 32) * w["m.norm"] * torch.sigmoid(x @ w["m.g"].T)) @ w["m.o"].T
    assert float((want[0] - lifted[0]).norm()) > 0.2 * float(lifted[0].norm())
    engine = PartEngine([part], torch.float32, DEV, 8)
    for sizes in ([120], [1], [64, 56], [2]):
        check(engine.run_cut("a", x, sizes)[0], want, torch.float32)


def test_the_memories_remember_and_the_next_request_starts_from_zero():
    """Slow decays: an early token still weighs hundreds of tokens later; a slot used again starts from zeros."""
    for part, m, kind in ((*mlstm_part(2, 16, 24, 15.0), "mlstm"), (*lightning_part(16, 24, [0.999, 0.9995]), "lightning")):
        w = random_weights(part, 3, scale={"i": 0.2, "f": 0.1})
        if kind == "mlstm":
            w["m.f.b"], w["m.i.b"] = torch.full((2,), 9.0), torch.full((2,), 0.5)
        load_part(part, w, torch.float32, DEV)
        x = torch.randn(400, 48, generator=torch.Generator().manual_seed(5))
        want = plain.MIXERS[kind](x, w, "m.", m, EPS)
        forgot = plain.MIXERS[kind](torch.cat([x[:3] * 0, x[3:]]), w, "m.", m, EPS)
        assert float((want[-1] - forgot[-1]).norm()) > 0.005 * float(want[-1].norm())
        engine = PartEngine([part], torch.float32, DEV, 8, max_requests=1)
        for _ in range(2):                       # the second time in the same slot
            check(engine.run_cut("a", x, [300] + [1] * 100)[0], want, torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,groups,normaliser", [(48, 1, False), (48, 6, True), (96, 3, True), (2048, 2, True), (5000, 1, False), (9000, 3, True)])
def test_norm_and_sigmoid_gate(dtype, width, groups, normaliser):
    gen = torch.Generator().manual_seed(width)
    y, rows, w = torch.randn(5, width, generator=gen), torch.randn(5, width + 7, generator=gen), torch.randn(width, generator=gen)
    y[:, :width // groups] *= 20                                    # parts of unlike sizes
    den = torch.randn(5, groups, generator=gen) if normaliser else None
    floor = torch.rand(5, groups, generator=gen) if normaliser else None
    for shift in (7, 4):                                            # rows that do not and that do start at multiples of 16 bytes
        z = rows[:, shift:shift + width]
        out = torch.zeros(5, width + shift, dtype=dtype, device=DEV)
        ops.norm_sigmoid_gate(y.to(DEV), rows.to(DEV)[:, shift:shift + width], w.to(DEV), groups, 1e-3, 0.7, out[:, shift:],
                              den.to(DEV) if normaliser else None, floor.to(DEV) if normaliser else None)
        u = y.view(5, groups, -1)
        if normaliser:
            u = u / (torch.maximum(den.abs(), floor) + 1e-6)[:, :, None]
        check(out[:, shift:], 0.7 * plain.rms(u, 1e-3).reshape(5, width) * w * torch.sigmoid(z), dtype)
        assert not bool(out[:, :shift].any())


# ------------------------------------------------------------------------------------------ feed-forwards
def experts_part(experts, top, ff, shared, width=64):
    return build_part("feed_forward", PartSpec("routed_experts", {
        "hidden_size": width, "num_experts": experts, "top": top, "expert_size": ff, "shared_size": shared, "alpha": 1.0,
        "shift": 0.0, "router_bias": True, "shared_gate": shared is not None, "suffix": ""}), prefix="f")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("experts,top,ff,shared,rows,width", [
    (8, 2, 40, 24, 1, 64), (8, 2, 40, None, 37, 64), (5, 5, 24, 56, 70, 64), (4, 1, 64, 8, 300, 64), (16, 3, 136, 32, 530, 96),
    (6, 2, 20, 12, 33, 76), (3, 2, 21, 7, 40, 50), (70, 4, 16, 16, 90, 64), (1, 1, 16, 16, 20, 64)])
def test_experts_behind_a_biased_router_and_a_gated_shared_one(dtype, experts, top, ff, shared, rows, width):
    part = experts_part(experts, top, ff, shared, width)
    w = random_weights(part, experts + rows, scale={"router": 0.3, "b": 1.0, "sg": 0.3})
    load_part(part, w, dtype, DEV)
    x = rounded(torch.randn(rows, width, generator=torch.Generator().manual_seed(rows)), dtype)
    mlp = {"router": {"top": top}, "shared": {"ff": shared} if shared else None}
    margins = []
    want = plain.experts(x, w, "f.", mlp, margins)
    clear = margins[0] > 1e-4                                    # x is exact in both, so only float32 ties are left out
    assert float(clear.float().mean()) > 0.95
    got = part.forward(x.to(dtype).to(DEV))
    got = got.materialize() if hasattr(got, "materialize") else got
    check(got[clear.to(DEV)], want[clear], dtype)


def test_the_routers_bias_moves_the_choice_and_the_weights():
    part = experts_part(6, 2, 16, 24)
    w = random_weights(part, 2, scale={"router": 0.1})
    w["f.router.b"] = torch.tensor([-9.0, 2.5, -7.0, 3.0, -30.0, -8.0])
    load_part(part, w, torch.float32, DEV)
    x = torch.randn(20, 64, generator=torch.Generator().manual_seed(1))
    gate = torch.empty(20, device=DEV)
    chosen, weight = ops.moe_route(x.to(DEV), part.router, 2, 1, 1, "softmax", True, None, part.router_bias, gate)
    assert sorted(set(chosen.cpu().flatten().tolist())) == [1, 3]
    want_chosen, want_weight, _ = plain.route(x, w, "f.", 2)
    assert torch.equal(chosen.cpu().long(), want_chosen)
    torch.testing.assert_close(weight.cpu(), want_weight, rtol=1e-5, atol=1e-6)
    torch.testing.assert_close(gate.cpu(), torch.sigmoid(x @ w["f.shared.sg"].T)[:, 0], rtol=1e-5, atol=1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,ff,rows", [(64, 48, 1), (64, 40, 30), (96, 256, 200), (76, 21, 33), (128, 512, 700)])
def test_dense_with_a_squared_relu(dtype, width, ff, rows):
    part = build_part("feed_forward", PartSpec("activated", {"hidden_size": width, "intermediate_size": ff,
                                                             "activation": "squared_relu", "bias": False, "suffix": ""}), prefix="f")
    w = random_weights(part, ff)
    assert set(w) == {"f.up", "f.down"}
    load_part(part, w, dtype, DEV)
    x = rounded(torch.randn(rows, width, generator=torch.Generator().manual_seed(rows)), dtype)
    got = part.forward(x.to(dtype).to(DEV))
    check(got.materialize() if hasattr(got, "materialize") else got, plain.dense(x, w, "f."), dtype)


# ------------------------------------------------------------------------------------------ the layer
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 8), (3, 7), (17, 100), (5, 1030), (2, 2048), (3, 5000), (2, 9001)])
def test_the_norm_of_the_sum(dtype, rows, width):
    gen = torch.Generator().manual_seed(width)
    h, y = torch.randn(rows, width, generator=gen), rounded(torch.randn(rows, width, generator=gen) * 2, dtype)
    scale, w = torch.randn(width, generator=gen), torch.randn(width, generator=gen)
    want = plain.norm_after(h, y, scale, 2.7, w, 1e-3)
    for copy in (True, False):
        on_device = h.to(DEV)
        out = ops.join_norm(on_device, y.to(dtype).to(DEV), scale.to(DEV), 2.7, w.to(DEV), 1e-3, copy)
        torch.testing.assert_close(on_device.cpu(), want, rtol=1e-5, atol=1e-5)
        assert (out is None) != copy
        if copy:
            assert torch.equal(out, on_device.to(torch.bfloat16))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("alpha,scaled,fed", [(2.5, True, True), (1.0, True, False), (0.4, False, True)])
def test_layers_that_norm_the_sum(dtype, alpha, scaled, fed):
    """Two layers one after another: the second reads the first one's rows as the first left them."""
    norm = {"hidden_size": 64, "eps": EPS}
    blocks = [build_part("block", PartSpec("sum_norm", {
        "mixer": PartSpec("lightning_attention", {"hidden_size": 64, "num_heads": 2, "key_dim": 16, "value_dim": 24, "decay": (0.6, 0.95),
                                                  "eps": EPS, "suffix": ""}),
        "feed_forward": PartSpec("activated", {"hidden_size": 64, "intermediate_size": 48, "activation": "squared_relu", "bias": False,
                                               "suffix": ""}) if fed else None,
        "mixer_norm": PartSpec("rmsnorm", {**norm, "tensor": "norm1"}), "ffn_norm": PartSpec("rmsnorm", {**norm, "tensor": "norm2"}),
        "width": 64, "alpha": alpha, "names": {"mixer_norm": "", "ffn_norm": "", "mixer": "mix", "feed_forward": "mlp",
                                               "mixer_scale": "ls1" if scaled else None, "ffn_scale": "ls2" if scaled else None}}),
        prefix=f"l{n}") for n in range(2)]
    x = torch.randn(30, 64, generator=torch.Generator().manual_seed(22))
    want, one = x, torch.ones(64)
    for n, block in enumerate(blocks):
        w = random_weights(block, 21 + n, scale={"ls1": 0.5, "ls2": 0.5})
        assert any(name.endswith("ls1") for name in w) == scaled and any(name.endswith("ls2") for name in w) == (scaled and fed)
        load_part(block, w, dtype, DEV)
        m = {"heads": 2, "dim": 16, "vdim": 24, "decay": [0.6, 0.95]}
        want = plain.norm_after(want, plain.lightning(want, w, f"l{n}.mix.", m, EPS), w.get(f"l{n}.ls1", one), alpha, w[f"l{n}.norm1"], EPS)
        if fed:
            want = plain.norm_after(want, plain.dense(want, w, f"l{n}.mlp."), w.get(f"l{n}.ls2", one), alpha, w[f"l{n}.norm2"], EPS)

    class Layers:                            # what the harness runs as a mixer
        entry_split = None

        def cache_spec(self):
            return blocks[0].cache_spec()

        def forward(self, rows, step, cache):
            stream = ResidualStream(x.to(DEV))
            for block in blocks:
                block.forward(stream, step, cache)
                cache.state.zero_()
            return stream.settle()
    got = PartEngine([Layers()], dtype, DEV, 8).run_cut("a", x, [30])[0]
    check(got, want, dtype)
