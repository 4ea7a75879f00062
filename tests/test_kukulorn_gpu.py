"""Kukulorn on the GPU: each new kernel (and each kernel that took a new option) against its plain reference; kept tokens,
windows, capped scores and gates in every attention kernel; the whole model in float32 and bfloat16 through replay (every way
of cutting, pages and slots used again), with a loud token far back, in long decoding, in batches against each request alone,
through the entry point with captured decode steps, and through the replay program itself."""
import json
import math
import os
import subprocess

import numpy as np
import pytest
import torch

import plain_kukulorn as plain
import replay_cases as rc
from kukulorn_cases import CONFIGS, PAGE_SIZE, long_memory, prompts, random_weights, write_folder
from torch_ops import TorchOps
from velox_amd import Engine, EngineConfig, Request, SamplingParams
from velox_amd.engine.batch import Workspace
from velox_amd.engine.replay import Replayer
from velox_amd.kernels import KernelError
from velox_amd.parts.base import NormedSum, SumOf

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = {"float32": dict(rtol=2e-4, atol=3e-5), "bfloat16": dict(rtol=6e-2, atol=6e-2)}
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}


@pytest.fixture(scope="module")
def ops():
    from velox_amd.kernels import load_ops

    return load_ops("cuda")


def close(got, want, dtype, scale=1.0):
    tol = TOL[dtype]
    torch.testing.assert_close(got.float().cpu(), want.float().cpu(), rtol=tol["rtol"], atol=tol["atol"] * scale)


def near(got, want, rel, what=""):
    """The largest difference, relative to the largest value."""
    err = float((got.float() - want.float()).abs().max()) / max(1e-6, float(want.float().abs().max()))
    assert err <= rel, f"{what}: {err}"


def ints(values):
    return torch.tensor(values, dtype=torch.int32).cuda()


# ----------------------------------------------------------------------------------------------------
# kernels alone
# ----------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("hidden", [6, 72, 321, 2048, 5120, 12288])
def test_terms_with_norms_of_their_own_and_the_norm_that_reads_the_sum(ops, dtype, hidden):
    """One or two normed terms beside a plain one or none, tensors and partial sums; chosen rows change nothing; the rows
    joined for the product before a pass, from every form of delta, clear the residual."""
    ref, dt = TorchOps(), DTYPES[dtype]
    for tokens in (3, 70):
        weights = tuple((1 + 0.2 * torch.randn(hidden)).cuda() for _ in range(2))
        outer = (1 + 0.1 * torch.randn(hidden)).cuda()
        residual, start = (torch.randn(tokens, hidden) * 2).cuda(), torch.randn(tokens, hidden).to(dt).cuda()
        a, b, p = (torch.randn(tokens, hidden).to(dt).cuda() * s for s in (3.0, 0.2, 1.0))
        sums = torch.randn(3, tokens, hidden).cuda()
        deltas = [NormedSum((a, b), weights, (0.5, 0.25), 1e-3, p), NormedSum((sums, b), weights, (0.5, 0.5), 1e-5, sums), NormedSum((a,), weights[:1], (2.0,), 1e-5)]
        rows = ints([tokens - 1, 0, 1])
        for delta in deltas:
            mine, theirs = residual.clone(), residual.clone()
            close(ops.normed_sum_norm(mine, delta, outer, 1e-5, dt, rows=rows), ref.normed_sum_norm(theirs, delta, outer, 1e-5, dt, rows=rows), dtype, 0.3)
            assert torch.equal(mine, residual)
            got, want = ops.normed_sum_norm(mine, delta, outer, 1e-5, dt), ref.normed_sum_norm(theirs, delta, outer, 1e-5, dt)
            torch.testing.assert_close(mine, theirs, rtol=1e-5, atol=1e-5)
            close(got, want, dtype, 0.3)
        for delta in deltas + [None, a, sums, SumOf(sums, p), SumOf(a, p)]:
            mine, theirs = residual.clone(), residual.clone()
            got, want = ops.join_rows(mine, delta, start, dt), ref.join_rows(theirs, delta, start, dt)
            assert not mine.any()
            close(got, want, dtype, 0.3)
            assert torch.equal(got[:, hidden:], start)
    kept = ops.kept_copy(residual, dt)
    assert kept.dtype == dt and kept.data_ptr() != residual.data_ptr()
    close(kept, residual, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("channels,first,extra,taps", [(20, 5, 3, 4), (64, 32, 0, 2), (7, 0, 1, 1), (300, 33, 40, 5), (96, 64, 8, 8)])
def test_convolution_of_inner_columns_with_a_bias(ops, dtype, channels, first, extra, taps):
    ref, dt = TorchOps(), DTYPES[dtype]
    weight, bias = torch.randn(channels, taps).cuda(), torch.randn(channels).cuda()
    tails = [torch.randn(5, taps - 1, channels).to(dt).cuda()] if taps > 1 else [None]
    tails.append(tails[0].clone() if taps > 1 else None)
    for lengths, slots in (((20, 1, 33), (3, 0, 2)), ((1, 1, 1), (2, 3, 0)), ((2, 1, 3), (0, 3, 1))):
        cu, slot = ints([0] + list(np.cumsum(lengths))), ints(slots)
        x = torch.randn(sum(lengths), first + channels + extra).to(dt).cuda()
        args = (channels, weight)
        got = ops.short_conv(x, *args, tails[0], slot, cu, max(lengths), activation="silu", first=first, bias=bias)
        want = ref.short_conv(x, *args, tails[1], slot, cu, max(lengths), activation="silu", first=first, bias=bias)
        close(got, want, dtype, 0.3)
        if taps > 1:
            assert torch.equal(tails[0], tails[1])


STATE_SPACES = [(3, 1, 10, 12), (4, 2, 16, 10), (2, 2, 6, 20), (3, 3, 9, 7), (2, 1, 160, 80), (4, 2, 64, 32), (1, 1, 1, 48), (4, 1, 128, 64), (2, 1, 300, 33), (1, 1, 700, 8), (2, 2, 33, 130)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads,groups,size,vdim", STATE_SPACES)
def test_state_space_kernels(ops, dtype, heads, groups, size, vdim):
    """Token by token and in chunks (full, partly filled, of one token) against the plain reference: portions of several
    sequences, single tokens, from states that other slots must not see; step sizes from nearly 0 to large, decays from "gone
    at once" to "kept"; then the head norm over equal parts."""
    ref, dt = TorchOps(), DTYPES[dtype]
    inner, gn = heads * vdim, groups * size
    rate, skip = torch.exp(1.5 * torch.randn(heads)).cuda(), torch.randn(heads).cuda()
    dt_bias = (-2.0 + 2.0 * torch.randn(heads)).cuda()
    first = torch.randn(5, heads, size, vdim).cuda() * 0.3
    for chunked in (False, True):
        states = [first.clone(), first.clone()]
        for lengths, slots in (((20, 1, 33, 200), (3, 0, 2, 1)), ((1, 1, 1, 1), (1, 3, 0, 2)), ((2, 64, 1), (0, 3, 1)), ((65, 128), (2, 0))):
            tokens = sum(lengths)
            cu, slot = ints([0] + list(np.cumsum(lengths))), ints(slots)
            xbc = torch.randn(tokens, inner + 2 * gn).to(dt).cuda()
            source = (2.0 * torch.randn(tokens, heads + 5)).to(dt).cuda()
            got, want = (o.state_space_scan(xbc, source, 3, dt_bias, rate, skip, state, slot, cu, max(lengths), heads, groups, size, vdim, **kw)
                         for o, state, kw in ((ops, states[0], dict(chunked=chunked)), (ref, states[1], {})))
            near(got, want, 2e-5, f"read-out {lengths} chunked={chunked}")
            near(states[0], states[1], 2e-5, f"state {lengths} chunked={chunked}")
        assert torch.equal(states[0][4], first[4])  # (a slot nobody holds is left alone)
    gate = torch.randn(tokens, inner + 9).to(dt).cuda()
    weight = (1 + 0.2 * torch.randn(inner)).cuda()
    for at in (0, 4, 7):
        for parts in {1, heads, vdim}:
            near(ops.gated_group_norm(want, gate, at, weight, 1e-5, parts, dt), ref.gated_group_norm(want, gate, at, weight, 1e-5, parts, dt),
                 1e-5 if dtype == "float32" else 1e-2, f"norm in {parts} parts")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width,parts", [(8192, 1), (6000, 2), (20000, 1), (18, 6), (2048, 8)])
def test_norm_of_a_gated_row_in_equal_parts(ops, dtype, width, parts):
    ref, dt = TorchOps(), DTYPES[dtype]
    read, gate, weight = torch.randn(9, width).cuda(), torch.randn(9, width + 8).to(dt).cuda(), (1 + 0.2 * torch.randn(width)).cuda()
    near(ops.gated_group_norm(read, gate, 8, weight, 1e-5, parts, dt), ref.gated_group_norm(read, gate, 8, weight, 1e-5, parts, dt), 1e-5 if dtype == "float32" else 1e-2)


@pytest.mark.parametrize("heads,groups,size,vdim", [(2, 1, 128, 64), (3, 1, 20, 12), (1, 1, 200, 100)])
def test_a_long_portion_of_the_state_space_equals_its_pieces_and_keeps_its_first_token(ops, heads, groups, size, vdim):
    """600 tokens in one step, in pieces that end inside and at a chunk's border, and token by token; decays that wipe the
    state out in between change nothing of the agreement, and with slow ones the loud first token still decides the end."""
    g = torch.Generator().manual_seed(size)
    n, inner, gn = 600, heads * vdim, groups * size
    xbc = torch.randn(n, inner + 2 * gn, generator=g)
    xbc[0, :inner] *= 300.0
    xbc[1:, inner:inner + gn] *= 0.3
    xbc = xbc.cuda()
    skip, bias = torch.ones(heads).cuda(), torch.zeros(heads).cuda()
    source = torch.full((n, heads), -1.0).cuda()

    def run(cuts, rows, steps, rate, **kw):
        state, outs, at = torch.zeros(2, heads, size, vdim).cuda(), [], 0
        for c in cuts:
            outs.append(ops.state_space_scan(rows[at:at + c].clone(), steps[at:at + c].clone(), 0, bias, rate, skip, state, ints([1]), ints([0, c]), c, heads, groups, size, vdim, **kw))
            at += c
        return torch.cat(outs), state

    abrupt = source.clone()
    abrupt[70::50] = 60.0  # (with the fast rate: a decay far below what float32 can hold)
    for steps, rate in ((source, torch.full((heads,), 1e-3).cuda()), (abrupt, torch.full((heads,), 20.0).cuda())):
        whole, state = run((n,), xbc, steps, rate)
        assert torch.equal(whole, run((n,), xbc, steps, rate)[0]) and bool(torch.isfinite(whole).all())
        for cuts, kw in (((n,), dict(chunked=False)), ((1, 2, 300, 17, 280), {}), ((64, 128, 63, 345), {}), ((63, 65, 472), dict(chunked=True))):
            pieces, piece_state = run(cuts, xbc, steps, rate, **kw)
            near(pieces, whole, 3e-5, f"pieces {cuts}")
            near(piece_state, state, 3e-5, f"state {cuts}")
    quiet = xbc.clone()
    quiet[0, :inner] = 0.0
    slow = torch.full((heads,), 1e-3).cuda()
    whole = run((n,), xbc, source, slow)[0]
    assert float((run((n,), quiet, source, slow)[0][-1] - whole[-1]).abs().max()) > 0.2 * float(whole[-1].abs().max())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("tokens,width,inter", [(1, 128, 192), (9, 64, 40), (16, 256, 96), (40, 128, 64), (90, 86, 22), (3, 41, 9)])
def test_rectified_gate_and_capped_logits(ops, dtype, tokens, width, inter):
    ref, dt = TorchOps(), DTYPES[dtype]
    x, weight = torch.randn(tokens, width).to(dt).cuda(), (torch.randn(2 * inter, width) / math.sqrt(width)).to(dt).cuda()
    want = ref.gated_act_mul(ref.linear(x, weight, None, torch.float32), "relu")
    for operand in (weight, ops.prepare_weight(weight, stacked=2)):
        if operand is not None:
            close(ops.linear_gated_act(x, operand, dt, "relu"), want, dtype, 0.5)
    logits = (torch.randn(tokens, inter) * 40).cuda()
    close(ops.softcap_(logits.clone(), 15.0), ref.softcap_(logits.clone(), 15.0), "float32")
    close(ops.softcap_(logits.clone(), 3.0, 0.25), 3.0 * torch.tanh(logits.double() * 0.25 / 3.0), "float32")


def _paged_case(nh, nkv, d, q_lens, kv_lens, page, dt, seed=0):
    g = torch.Generator().manual_seed(seed)
    need = [(n + page - 1) // page for n in kv_lens]
    pages = sum(need) + 1
    k_cache = torch.randn(pages, nkv, page, d, generator=g).to(dt).cuda()
    v_cache = torch.randn(pages, nkv, d, page, generator=g).to(dt).cuda()
    tables = torch.zeros(len(kv_lens), max(need), dtype=torch.int32)
    perm = torch.randperm(pages - 1, generator=g) + 1
    at = 0
    for b, n in enumerate(need):
        tables[b, :n] = perm[at:at + n]
        at += n
    cu = ints([0] + list(np.cumsum(q_lens)))
    q = (torch.randn(sum(q_lens), nh * d, generator=g) * 0.5).to(dt).cuda()
    return q, k_cache, v_cache, tables.cuda(), cu, ints(kv_lens)


ATTENTION_CASES = [
    (4, 2, 64, 24, [1, 1, 1], [70, 1, 300]),             # single tokens
    (8, 1, 64, 1500, [1, 1], [5000, 2300]),              # single tokens whose keys are split over workgroups and merged
    (4, 2, 64, 17, [9, 30, 2], [9, 155, 40]),            # short portions
    (8, 2, 64, 136, [600, 500], [600, 1500]),            # long portions
    (28, 4, 64, 200, [700, 300], [900, 2700]),           # long portions in the kernel whose tiles are loaded straight into LDS
    (16, 4, 128, 100, [300], [900]),
    (20, 1, 32, 40, [1, 1, 40, 7], [800, 3, 100, 7]),    # more query heads to a key head than one tile of rows; single tokens before portions
    (2, 1, 16, 5, [1, 1, 3, 50], [40, 9, 30, 50]),
    (3, 1, 272, 50, [1, 9, 30], [70, 9, 155]),           # beyond the tiled kernels
]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("nh,nkv,d,window,q_lens,kv_lens", ATTENTION_CASES)
@pytest.mark.parametrize("keep,page", [(6, 16), (16, 16), (17, 8), (70, 32), (3, 4), (40, 128)])
def test_loud_keys_at_the_edges_of_a_window_and_of_the_kept_tokens(ops, dtype, nh, nkv, d, window, q_lens, kv_lens, keep, page):
    """The last query's last kept token, the one behind it, the first token of its window and the one before it are made loud
    in turn: the kept one and the window's change that query's result, the others do not, and all equal the reference.  The
    bias by distance and a gate per head are there too."""
    ref, dt = TorchOps(), DTYPES[dtype]
    bias = torch.randn(nh, 30).cuda()
    gate = torch.randn(sum(q_lens), nh + 3).to(dt).cuda()
    prefix = next((i for i, n in enumerate(q_lens) if n != 1), len(q_lens))
    longest = max(range(len(kv_lens)), key=lambda b: kv_lens[b])
    last_row, last = sum(q_lens[:longest + 1]) - 1, kv_lens[longest] - 1
    results = {}
    for label, place in (("plain", None), ("kept", keep - 1), ("behind", keep), ("inside", last - window + 1), ("outside", last - window)):
        q, k_cache, v_cache, tables, cu, lens = _paged_case(nh, nkv, d, q_lens, kv_lens, page, dt)
        if place is not None and not 0 <= place <= last:
            continue
        if place is not None:
            page_id, offset = int(tables[longest, place // page]), place % page
            for g in range(nkv):  # along the last query of the group's first head
                k_cache[page_id, g, offset] = 40.0 * torch.nn.functional.normalize(q[last_row].view(nh, d)[g * (nh // nkv)].float(), dim=0).to(dt)
            v_cache[page_id, :, :, offset] = 5.0
        args = (q, nh, nkv, d, k_cache, v_cache, page, tables, cu, lens, max(q_lens), max(kv_lens), 1.0 / math.sqrt(d), window, max(q_lens) == 1, Workspace(torch.device("cuda")))
        extra = dict(distance_bias=bias, keep_first=keep, gate=(gate, 2, 0))
        got = ops.paged_attention(*args, decode_prefix=prefix, **extra)
        close(got, ref.paged_attention(*args, **extra), dtype)
        results[label] = got[last_row].view(nh, d)[0].float() / torch.sigmoid(gate[last_row, 2].float())
    seen = lambda place: place > last - window or place < keep  # noqa: E731
    for label, place in (("kept", keep - 1), ("behind", keep), ("inside", last - window + 1), ("outside", last - window)):
        if label in results and place <= last:
            if seen(place):
                assert float((results[label] - results["plain"]).abs().max()) > 1.0, label
            else:
                assert torch.equal(results[label], results["plain"]), label


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("nh,nkv,d,window,q_lens,kv_lens", ATTENTION_CASES)
@pytest.mark.parametrize("channels", [None, 0, 11, -1])
def test_capped_scores_and_gates(ops, dtype, nh, nkv, d, window, q_lens, kv_lens, channels):
    """Scores far beyond the cap and far below it; no gate, one per head, one per channel of a part of the head, of all of it."""
    ref, dt = TorchOps(), DTYPES[dtype]
    prefix = next((i for i, n in enumerate(q_lens) if n != 1), len(q_lens))
    q, k_cache, v_cache, tables, cu, lens = _paged_case(nh, nkv, d, q_lens, kv_lens, 16, dt)
    q = q * 6
    gate = None
    if channels is not None:
        channels = d if channels < 0 else channels
        gate = (torch.randn(sum(q_lens), nh * max(channels, 1) + 8).to(dt).cuda(), 4, channels)
    args = (q, nh, nkv, d, k_cache, v_cache, 16, tables, cu, lens, max(q_lens), max(kv_lens), 1.0 / math.sqrt(d), None, max(q_lens) == 1, Workspace(torch.device("cuda")))
    got = ops.paged_attention(*args, decode_prefix=prefix, softcap=2.5, gate=gate)
    want = ref.paged_attention(*args, softcap=2.5, gate=gate)
    close(got, want, dtype)
    plain_scores = ops.paged_attention(*args, decode_prefix=prefix, gate=gate) if gate is None else None
    if plain_scores is not None and max(kv_lens) > 20:
        assert float((plain_scores.float() - got.float()).abs().max()) > 0.1
    with pytest.raises(KernelError):
        ops.paged_attention(*args, softcap=-1.0)


# ----------------------------------------------------------------------------------------------------
# the whole model
# ----------------------------------------------------------------------------------------------------
def rows_close(got, want, dtype, label, limit=0.05, share=0.9):
    if dtype == "float32":  # (rounding grows with the largest logit of a row, of which the small ones are differences)
        torch.testing.assert_close(got, want, msg=lambda m: f"{label}: {m}", rtol=2e-4, atol=3e-5 * max(1.0, float(want.abs().max())))
    else:
        # a row's root mean square error beside the row's root mean square; sharp weights that run several times make a few places
        # sensitive to any rounding (the plain model with its weights changed by 0.2% moves by a tenth there), so few may exceed the limit
        err = (got - want).square().mean(-1).sqrt() / want.square().mean(-1).sqrt()
        assert float((err < limit).float().mean()) >= share and float(err.median()) < 0.025, f"{label}: {err}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C", "D", "E"])
def test_all_ways_of_cutting_on_the_gpu(tmp_path, name, dtype):
    folder = write_folder(tmp_path / name, CONFIGS[name], seed=2, dtype=dtype)
    config, weights = plain.read_folder(folder)
    requests = prompts(config["vocab"], [141, 1, 37, 98, 2, 64, 75], seed=11)
    expected = {rid: plain.forward(config, weights, tokens).float() for rid, tokens in requests.items()}
    page = PAGE_SIZE[name]
    results = {}
    for label, trace in (("whole", rc.whole(requests)), ("tail", rc.tail_one_by_one(requests)), ("portions", rc.changing_portions(requests)),
                         ("mixed", rc.mixed(requests, seed=5)), ("recompute", rc.mixed(requests, seed=8, preempt=("r0", "r3", "r6")))):
        replayer = Replayer(folder, dtype, rc.tokens_needed(trace, page), block_size=page, max_live=4)
        outputs = rc.run_trace(replayer, trace)
        results[label] = rc.collect(trace, outputs, requests)
        for rid in requests:
            rows_close(results[label][rid], expected[rid], dtype, f"{name} {label} {rid}")
        if label in ("mixed", "recompute"):
            assert sum((len(t) + page - 1) // page for t in requests.values()) > replayer.cache.num_total_pages
    if dtype == "float32":
        for label in ("tail", "portions", "mixed", "recompute"):  # the ways of cutting agree with each other
            for rid in requests:
                rows_close(results[label][rid], results["whole"][rid], dtype, f"{name} {label} beside whole {rid}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("far_at,length", [(0, 600), (3, 200), (15, 200), (16, 200), (19, 200), (20, 200), (64, 200)])
def test_a_loud_token_far_back(tmp_path, dtype, far_at, length):
    """One early token is made loud and the states keep for long: hundreds of tokens on, far behind every window, the logits
    still depend on it (through the states, the layers that see all keys and, below twenty, the kept tokens) and equal the
    plain model's, from a portion and from single tokens, written by one step and read by later ones."""
    config = CONFIGS["C"]
    weights = long_memory(random_weights(config, 9))
    tokens = [t if t != 159 else 158 for t in prompts(config["vocab"], [length], seed=5)["r0"]]
    tokens[far_at] = 159
    weights["embed"][159] *= 4.0
    folder = write_folder(tmp_path / "far", config, seed=9, dtype=dtype, weights=weights)
    config, weights = plain.read_folder(folder)
    right = plain.forward(config, weights, tokens)
    other = list(tokens)
    other[far_at] = 5
    moved = (right[-30:] - plain.forward(config, weights, other)[-30:]).abs().amax(-1)
    assert float(moved.median()) > 0.02
    requests = {"r0": tokens}
    cuts = (far_at + 1, 2, 100, 1, 3, 33, 2)
    for label, trace in (("whole", rc.whole(requests)), ("tail", rc.tail_one_by_one(requests, tail=40)), ("portions", rc.changing_portions(requests, sizes=cuts))):
        replayer = Replayer(folder, dtype, length + 16, block_size=16, max_live=2)
        got = rc.collect(trace, rc.run_trace(replayer, trace), requests)
        rows_close(got["r0"][-150:], right[-150:].float(), dtype, f"far {label}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_and_a_batch_against_each_request_alone(tmp_path, dtype):
    """A prompt of a few tokens, then 200 tokens one by one across many page borders (the windows pass over decoded tokens, the
    kept tokens were partly decoded); then four requests of unequal length decoded together, whose logits equal those of each
    request decoded alone."""
    folder = write_folder(tmp_path / "C", CONFIGS["C"], seed=4, dtype=dtype)
    config, weights = plain.read_folder(folder)
    tokens = prompts(config["vocab"], [205], seed=12)["r0"]
    want = plain.forward(config, weights, tokens).float()
    replayer = Replayer(folder, dtype, 4 * 224, block_size=16, max_live=4)
    rows = [replayer.step({"step": 0, "entries": [{"id": "x", "tokens": tokens[:5], "want": [0, 4]}], "end": []})]
    for i in range(5, 205):
        rows.append(replayer.step({"step": i, "entries": [{"id": "x", "tokens": [tokens[i]], "want": [0]}], "end": ["x"] if i == 204 else []}))
    rows_close(torch.from_numpy(np.concatenate(rows)), want[[0] + list(range(4, 205))], dtype, "long decoding")
    texts = prompts(config["vocab"], [70, 9, 33, 120], seed=13)
    alone = {}
    for rid, text in texts.items():
        head = len(text) - 6
        replayer.step({"step": 0, "entries": [{"id": rid, "tokens": text[:head], "want": []}], "end": []})
        alone[rid] = [replayer.step({"step": 1, "entries": [{"id": rid, "tokens": [t], "want": [0]}], "end": []}) for t in text[head:]]
        replayer.step({"step": 2, "entries": [], "end": [rid]})
    replayer.step({"step": 0, "entries": [{"id": rid, "tokens": text[:len(text) - 6], "want": []} for rid, text in texts.items()], "end": []})
    for k in range(6):
        out = replayer.step({"step": 1 + k, "entries": [{"id": rid, "tokens": [text[len(text) - 6 + k]], "want": [0]} for rid, text in texts.items()], "end": []})
        for row, rid in zip(out, texts):
            rows_close(torch.from_numpy(row)[None], torch.from_numpy(alone[rid][k]), dtype, f"{rid} in a batch")


def test_captured_steps_equal_eager_ones(tmp_path):
    """Single tokens replayed from captured HIP graphs (padded rows, the state slot of the padding) against the same steps
    launched one kernel at a time, several replays with other work between them."""
    folder = write_folder(tmp_path / "C", CONFIGS["C"], seed=4, dtype="bfloat16")
    texts = prompts(CONFIGS["C"]["vocab"], [40, 9, 33], seed=13)
    outputs = []
    for graphs in (False, True):
        replayer = Replayer(folder, "bfloat16", 4 * 64, block_size=16, max_live=4, enable_graphs=graphs)
        assert replayer.runner.uses_graphs == graphs
        rows = []
        replayer.step({"step": 0, "entries": [{"id": rid, "tokens": text[:-5], "want": []} for rid, text in texts.items()], "end": []})
        for k in range(5):
            rows.append(replayer.step({"step": 1 + k, "entries": [{"id": rid, "tokens": [text[len(text) - 5 + k]], "want": [0]} for rid, text in texts.items()], "end": []}))
            replayer.step({"step": 10 + k, "entries": [{"id": "other", "tokens": [3, 4, 5][: 1 + k % 3], "want": []}], "end": ["other"]})
        outputs.append(np.concatenate(rows))
        if graphs:
            assert replayer.runner.num_graph_replays == 5
    np.testing.assert_allclose(outputs[1], outputs[0], rtol=2e-2, atol=2e-2)


@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation_through_the_entry_point(tmp_path, ops, graphs):
    """Scheduler, step function, captured decode steps (``graphs``) and sampler around the model, in float32: greedy tokens
    equal the plain model's, also when the pool is so small that requests wait for pages or are preempted."""
    folder = write_folder(tmp_path / "C", CONFIGS["C"], seed=6)
    config, weights = plain.read_folder(folder)
    texts = list(prompts(config["vocab"], [5, 19, 13, 40], seed=7).values())
    steps = 12

    def plain_greedy(prompt):
        tokens = list(prompt)
        for _ in range(steps):
            tokens.append(int(plain.forward(config, weights, tokens)[-1].argmax()))
        return tokens[len(prompt):]

    want = [plain_greedy(p) for p in texts]
    for pages in (64, 7):
        engine = Engine.from_pretrained(EngineConfig(model=folder, dtype="float32", device="cuda", max_model_len=96, max_num_seqs=4, max_num_batched_tokens=32,
                                                     max_prefill_chunk_size=11, block_size=16, num_gpu_blocks=pages, enable_cuda_graphs=graphs, seed=0), ops=ops)
        assert engine.runner.uses_graphs == graphs and engine.cache.prefix is None
        requests = [Request(f"r{i}", p, SamplingParams(temperature=0.0, max_tokens=steps, ignore_eos=True)) for i, p in enumerate(texts)]
        engine.generate(requests)
        assert [r.output_token_ids for r in requests] == want
        assert engine.cache.num_used_pages() == 0
        if graphs:
            assert engine.runner.num_graph_replays > 0


def test_the_replay_program_itself(tmp_path):
    folder = write_folder(tmp_path / "A", CONFIGS["A"], seed=9, dtype="bfloat16")
    config, weights = plain.read_folder(folder)
    tokens = prompts(config["vocab"], [30], seed=1)["r0"]
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": tokens[:17], "want": [0, 16]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": tokens[17:19], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": tokens[19:], "want": [10]}], "end": ["a"]}]
    for dtype in ("float32", "bfloat16"):
        out = tmp_path / f"out_{dtype}"
        done = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(out), "--max-tokens", "64"],
                              input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=600)
        assert done.returncode == 0, done.stderr[-2000:]
        assert [line for line in done.stdout.splitlines() if line.startswith("done")] == ["done 0", "done 1", "done 2"]
        assert not (out / "1.f32").exists()
        got = np.concatenate([np.fromfile(out / "0.f32", dtype="<f4").reshape(2, -1), np.fromfile(out / "2.f32", dtype="<f4").reshape(1, -1)])
        rows_close(torch.from_numpy(got), plain.forward(config, weights, tokens)[[0, 16, 29]].float(), dtype, "replay program")
