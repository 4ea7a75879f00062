"""Kedanex on the GPU: each new kernel (and each kernel that took a new option) against its plain reference; a loud key at a
window's edge in every attention kernel; the whole model in float32 and bfloat16 through replay (every way of cutting, pages
and slots used again), with a loud token far back, in long decoding, in batches against each request alone, through the
entry point with captured decode steps, and through the replay program itself."""
import json
import math
import os
import subprocess

import numpy as np
import pytest
import torch

import plain_kedanex as plain
import replay_cases as rc
from kedanex_cases import CONFIGS, PAGE_SIZE, long_memory, prompts, random_weights, write_folder
from torch_ops import TorchOps
from velox_amd import Engine, EngineConfig, Request, SamplingParams
from velox_amd.engine.batch import Workspace
from velox_amd.engine.replay import Replayer
from velox_amd.parts import make_part
from velox_amd.parts.base import OutputNormSink, ReadyInput, ResidualCopy

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
def test_a_norm_behind_and_a_norm_before(ops, dtype, hidden):
    ref, dt = TorchOps(), DTYPES[dtype]
    for tokens in (3, 70):
        inner, outer = (1 + 0.1 * torch.randn(hidden)).cuda(), (1 + 0.1 * torch.randn(hidden)).cuda()
        residual = (torch.randn(tokens, hidden) * 2).cuda()
        deltas = [torch.randn(tokens, hidden).to(dt).cuda() * 3]
        if hidden % 4 == 0:  # (partial sums are what products of such widths leave)
            deltas.append(torch.randn(3, tokens, hidden).cuda())
        for delta in deltas:
            mine, theirs = residual.clone(), residual.clone()
            rows = ints([tokens - 1, 0, 1])
            close(ops.norm_add_norm(mine, delta, inner, 1e-3, outer, 1e-5, dt, rows=rows), ref.norm_add_norm(theirs, delta, inner, 1e-3, outer, 1e-5, dt, rows=rows), dtype, 0.3)
            assert torch.equal(mine, residual)
            got, want = ops.norm_add_norm(mine, delta, inner, 1e-3, outer, 1e-5, dt), ref.norm_add_norm(theirs, delta, inner, 1e-3, outer, 1e-5, dt)
            torch.testing.assert_close(mine, theirs, rtol=1e-5, atol=1e-5)
            close(got, want, dtype, 0.3)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width", [1, 37, 96, 320, 8448, 33000])
def test_poly_norm(ops, dtype, width):
    ref, dt = TorchOps(), DTYPES[dtype]
    coefficients = torch.tensor([0.8, -0.6, 0.5, 0.3]).cuda()
    for tokens in (3, 90):
        x = (torch.randn(tokens, width) * torch.rand(tokens, 1) * 4).to(dt).cuda()
        close(ops.poly_norm(x, coefficients, 1e-5), ref.poly_norm(x, coefficients, 1e-5), dtype)


DELTAS = [(3, 12, 12, 5), (2, 64, 64, 16), (1, 128, 48, 24), (3, 6, 6, 3), (2, 20, 20, 7), (1, 48, 48, 1), (2, 72, 40, 8), (1, 256, 20, 32), (1, 512, 8, 64), (4, 32, 32, 40)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads,dim,vdim,rank", DELTAS)
def test_generalized_delta_rule_kernels(ops, dtype, heads, dim, vdim, rank):
    """Preparation, recurrence and head norm against the plain references: portions of several sequences (one of a single
    token) and then single tokens, from states that other slots must not see."""
    ref, dt = TorchOps(), DTYPES[dtype]
    ks, vs = heads * dim, heads * vdim
    width = 3 * ks + 2 * vs + rank
    at = dict(r=0, k=ks, v=2 * ks, a=2 * ks + vs, g=3 * ks + vs, low=3 * ks + 2 * vs)
    a_bias, w0 = torch.randn(ks).cuda(), torch.randn(ks).cuda() * 2
    w2 = (torch.randn(ks, rank) / math.sqrt(rank)).to(dt).cuda()
    weight = (1 + 0.2 * torch.randn(vs)).cuda()
    states = [torch.randn(4, heads, dim, vdim).cuda() * 0.3] * 2
    states = [states[0].clone(), states[0].clone()]
    kept = states[0].clone()
    for lengths, slots in (((20, 1, 33, 300), (3, 0, 2, 1)), ((1, 1, 1, 1), (1, 3, 0, 2)), ((2, 7, 1), (0, 3, 1))):
        tokens = sum(lengths)
        cu, slot = ints([0] + list(np.cumsum(lengths))), ints(slots)
        main = torch.randn(tokens, width).to(dt).cuda()
        got = ops.removal_prepare(main, at["r"], at["k"], at["a"], at["low"], rank, heads, dim, a_bias, w2, w0, math.exp(-0.5))
        want = ref.removal_prepare(main, at["r"], at["k"], at["a"], at["low"], rank, heads, dim, a_bias, w2, w0, math.exp(-0.5))
        for mine, theirs in zip(got, want):
            torch.testing.assert_close(mine, theirs, rtol=2e-5, atol=2e-6)
        reads = [o.linear_scan(want[0], main, at["v"], want[1], want[2], state, slot, cu, max(lengths), heads, heads, dim, vdim, "removal")
                 for o, state in ((ops, states[0]), (ref, states[1]))]
        near(reads[0], reads[1], 2e-5, "read-out")
        near(states[0], states[1], 2e-5, "state")
        a = ops.gated_head_norm(reads[1], weight, 1e-6, main, at["g"], "sigmoid", heads, vdim, dt)
        b = ref.gated_head_norm(reads[1], weight, 1e-6, main, at["g"], "sigmoid", heads, vdim, dt)
        near(a, b, 1e-5 if dtype == "float32" else 1e-2, "head norm")
    assert not torch.equal(states[0], kept)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads,dim,vdim,rank", [(2, 64, 64, 16), (1, 128, 48, 24), (3, 16, 20, 5), (2, 32, 7, 33), (1, 48, 48, 1), (5, 80, 80, 64), (1, 96, 33, 8), (1, 112, 16, 3)])
def test_chunks_of_tokens_equal_the_token_by_token_kernels(ops, dtype, heads, dim, vdim, rank):
    """Long and short portions beside single tokens (chunks that are full, partly filled, of one token), strong and weak decays,
    keys that come back unchanged, against the plain reference; then a loud first token that must still be read at the end
    of a long portion, whole and in pieces that end inside and at a chunk's border."""
    ref, dt = TorchOps(), DTYPES[dtype]
    ks, vs = heads * dim, heads * vdim
    width = 3 * ks + 2 * vs + rank
    at = (0, ks, 2 * ks, 2 * ks + vs, 3 * ks + 2 * vs)
    w2 = (torch.randn(ks, rank) * 2 / math.sqrt(rank)).to(dt).cuda()
    a_bias, w0 = torch.randn(ks).cuda() * 2, torch.randn(ks).cuda() * 3  # (decays from 0.545 to 1, removal rates from 0 to 1)
    states = [torch.randn(5, heads, dim, vdim).cuda() * 0.3]
    states.append(states[0].clone())
    kept = states[0].clone()
    for lengths, slots in (((100, 1, 16, 33), (3, 0, 2, 1)), ((17,), (2,)), ((1, 48, 15), (1, 3, 0)), ((300, 2), (0, 3))):
        cu, slot = ints([0] + list(np.cumsum(lengths))), ints(slots)
        main = torch.randn(sum(lengths), width)
        main[3::4, ks:2 * ks] = main[2::4, ks:2 * ks][: main[3::4].shape[0]]  # (every fourth key is the one before it)
        main = main.to(dt).cuda()
        got = ops.removal_scan(main, *at, rank, heads, dim, vdim, a_bias, w2, w0, math.exp(-0.5), states[0], slot, cu, max(lengths), chunked=True)
        want = ref.removal_scan(main, *at, rank, heads, dim, vdim, a_bias, w2, w0, math.exp(-0.5), states[1], slot, cu, max(lengths))
        near(got, want, 3e-5, "read-out")
        near(states[0], states[1], 3e-5, "state")
    assert torch.equal(states[0][4], kept[4])  # (a slot nobody holds is left alone)
    # a loud first token behind decays near 1 and removal rates near 0
    n = 500
    main = torch.randn(n, width)
    main[:, at[4]:] *= 0.2
    main[0, at[2]:at[2] + vs] *= 300.0
    main = main.to(dt).cuda()
    slow = torch.full((ks,), -8.0).cuda()

    def run(cuts, rows, **kw):
        state, outs, here = torch.zeros(2, heads, dim, vdim).cuda(), [], 0
        for c in cuts:
            outs.append(ops.removal_scan(rows[here:here + c].clone(), *at, rank, heads, dim, vdim, slow, w2 * 0.1, slow, math.exp(-0.5), state, ints([1]), ints([0, c]), c, **kw))
            here += c
        return torch.cat(outs), state

    whole, state = run((n,), main)
    assert torch.equal(whole, run((n,), main)[0])
    for cuts, kw in (((n,), dict(chunked=False)), ((1, 2, 300, 17, 180), {}), ((16, 32, 47, 405), {}), ((15, 33, 452), dict(chunked=True))):
        pieces, piece_state = run(cuts, main, **kw)
        near(pieces, whole, 3e-5, f"pieces {cuts}")
        near(piece_state, state, 3e-5, f"state {cuts}")
    quiet = main.clone()
    quiet[0, at[2]:at[2] + vs] = 0.0
    assert float((run((n,), quiet)[0][-1] - whole[-1]).abs().max()) > 0.2 * float(whole[-1].abs().max())


@pytest.mark.parametrize("heads,dim,vdim", [(2, 64, 64), (1, 128, 128), (3, 32, 48), (2, 12, 12), (1, 256, 16), (1, 72, 40)])
def test_a_long_portion_equals_its_pieces_and_its_first_token_is_kept(ops, heads, dim, vdim):
    """600 tokens in one step, in pieces (one of a single token, one of two) and against the plain loop; with decays close
    to 1 and small removal rates the loud first token's write still decides the last read-out."""
    ref = TorchOps()
    g = torch.Generator().manual_seed(dim)
    n = 600
    unit = torch.nn.functional.normalize(torch.randn(n, heads, dim, generator=g), dim=-1)
    vectors = torch.stack([torch.randn(n, heads, dim, generator=g), unit, 1e-3 * torch.rand(n, heads, dim, generator=g) * unit], 2).cuda().contiguous()
    values = torch.randn(n, heads * vdim, generator=g).cuda()
    values[0] *= 300.0
    decay = (1.0 - 2e-4 * torch.rand(n, heads * dim, generator=g)).cuda()
    lengths = (0.5 + torch.rand(n, heads, generator=g)).cuda()

    def run(operations, cuts, v):
        state, outs, at = torch.zeros(2, heads, dim, vdim).cuda(), [], 0
        for c in cuts:
            outs.append(operations.linear_scan(vectors[at:at + c].clone(), v[at:at + c].clone(), 0, decay[at:at + c].clone(), lengths[at:at + c].clone(), state,
                                               ints([1]), ints([0, c]), c, heads, heads, dim, vdim, "removal"))
            at += c
        return torch.cat(outs), state

    whole, state = run(ops, (n,), values)
    pieces, state_pieces = run(ops, (1, 2, 300, 17, 280), values)
    near(pieces, whole, 2e-5, "pieces")
    near(state_pieces, state, 2e-5, "state of the pieces")
    again, state_again = run(ops, (n,), values)
    assert torch.equal(whole, again) and torch.equal(state, state_again)
    want, want_state = run(ref, (n,), values)
    near(whole, want, 5e-5, "read-out")
    near(state, want_state, 5e-5, "state")
    quiet = values.clone()
    quiet[0] = 0.0
    assert float((run(ops, (n,), quiet)[0][-1] - whole[-1]).abs().max()) > 0.2 * float(whole[-1].abs().max())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width", [1, 20, 33, 192, 3072])
def test_gated_recurrence_in_pieces_and_in_single_tokens(ops, dtype, width):
    """Portions of unequal sequences (none, one and several pieces of the kernel's two passes, lengths at the pieces' borders),
    single tokens, slots that are used again; cut otherwise, the same results up to rounding."""
    ref, dt = TorchOps(), DTYPES[dtype]
    zb, xb = torch.randn(width).cuda() - 1, torch.randn(width).cuda()
    states = [torch.randn(5, width).cuda().abs()] * 2
    states = [states[0].clone(), states[0].clone()]
    kept = states[0].clone()
    for lengths, slots in (((200, 1, 65, 64), (3, 0, 2, 1)), ((1, 1, 1), (2, 3, 0)), ((2, 63, 1, 31), (0, 3, 1, 2)), ((32, 33), (1, 2)), ((500,), (0,))):
        cu, slot = ints([0] + list(np.cumsum(lengths))), ints(slots)
        rows = (torch.randn(sum(lengths), 3 * width) * 2).to(dt).cuda()
        got = ops.gated_scan(rows, width, zb, xb, 0.5, states[0], slot, cu, max(lengths))
        want = ref.gated_scan(rows, width, zb, xb, 0.5, states[1], slot, cu, max(lengths))
        close(got, want, dtype)
        torch.testing.assert_close(states[0], states[1], rtol=2e-5, atol=2e-6)
    assert torch.equal(states[0][4], kept[4])  # (a slot nobody holds is left alone)
    rows = (torch.randn(300, 3 * width) * 2).cuda()
    rows[:, :width] = 0.15 * rows[:, :width] - 6.0  # gates nearly closed: the first token stays
    rows[0, :width] = 6.0
    rows[0, width:2 * width] = 50.0
    outs = []
    for cuts in ((300,), (1, 2, 100, 64, 133), (31, 1, 268)):
        state, at, parts = torch.zeros(2, width).cuda(), 0, []
        for c in cuts:
            parts.append(ops.gated_scan(rows[at:at + c].clone(), width, zb * 0, xb, 0.5, state, ints([1]), ints([0, c]), c))
            at += c
        outs.append((torch.cat(parts), state))
    for out, state in outs[1:]:
        torch.testing.assert_close(out, outs[0][0], rtol=2e-5, atol=1e-5)
        torch.testing.assert_close(state, outs[0][1], rtol=2e-5, atol=1e-5)
    assert float(outs[0][1][1].min()) > 5.0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads,kv_heads,dim,half,tokens", [(4, 2, 16, 4, 11), (8, 1, 64, 32, 300), (3, 3, 10, 0, 5), (5, 1, 14, 3, 9), (2, 1, 272, 100, 7), (1, 1, 128, 64, 600)])
def test_rotation_then_norm_with_values_that_are_the_keys(ops, dtype, heads, kv_heads, dim, half, tokens):
    ref, dt = TorchOps(), DTYPES[dtype]
    cached = (dim + 15) // 16 * 16
    page, pages = 4, (tokens + 3) // 4 + 3
    rows = (torch.randn(tokens, (heads + kv_heads) * dim) * 3).to(dt).cuda()
    positions = torch.randint(0, 64, (tokens,), dtype=torch.int32).cuda()
    cos = sin = None
    if half:
        angles = torch.rand(64, half) * 6.0
        cos, sin = angles.cos().cuda(), angles.sin().cuda()
    slots = torch.randperm((pages - 1) * page)[:tokens].to(torch.int32).cuda() + page
    caches = [[torch.full((pages, kv_heads, page, cached), 9.0, dtype=dt).cuda(), torch.full((pages, kv_heads, cached, page), 9.0, dtype=dt).cuda()] for _ in range(2)]
    options = dict(post_norm_eps=1e-5, values_are_keys=True)
    got = ops.rotate_pad_write(rows, heads, kv_heads, dim, dim, cached, positions, cos, sin, slots, *caches[0], page, **options)
    want = ref.rotate_pad_write(rows, heads, kv_heads, dim, dim, cached, positions, cos, sin, slots, *caches[1], page, **options)
    close(got, want, dtype, 0.5)
    close(caches[0][0], caches[1][0], dtype, 0.5)
    assert torch.equal(caches[0][1], caches[1][1])  # (values: the keys as they stand in the rows)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("tokens,hidden,inter,experts,top", [(70, 64, 32, 4, 2), (9, 88, 20, 6, 3), (1, 256, 64, 12, 1), (300, 136, 72, 2, 2), (3, 41, 9, 3, 3)])
def test_experts_whose_last_kernel_takes_the_norm_behind_and_the_next(ops, dtype, tokens, hidden, inter, experts, top):
    ref, dt = TorchOps(), DTYPES[dtype]
    x = torch.randn(tokens, hidden).to(dt).cuda()
    gate_up = (torch.randn(experts * 2 * inter, hidden) / math.sqrt(hidden)).to(dt).cuda()
    down = (torch.randn(experts * hidden, inter) / math.sqrt(inter)).to(dt).cuda()
    logits = (torch.randn(tokens, experts) * 2).cuda()
    choice, weight = ops.route_top(logits, top, "softmax", True)
    want_choice, want_weight = plain.choose_experts(logits.cpu().double(), top)
    assert torch.equal(choice.cpu().long(), want_choice)
    torch.testing.assert_close(weight.cpu(), want_weight.float(), rtol=1e-5, atol=1e-6)
    following = make_part("norm", "rmsnorm", prefix="", hidden_size=hidden, eps=1e-4, weight_name="")
    following.weight = (1 + 0.1 * torch.randn(hidden)).cuda()
    behind = (1 + 0.1 * torch.randn(hidden)).cuda()
    residual = torch.randn(tokens, hidden).cuda()
    for follow in (following, None):
        mine, theirs = residual.clone(), residual.clone()
        got = ops.routed_experts(x, choice, weight, gate_up, down, experts, False, None, dt, Workspace(torch.device("cuda")), output_norm=OutputNormSink(mine, behind, 1e-5, 1.0, follow))
        want = ref.routed_experts(x, choice, weight, gate_up, down, experts, False, None, dt, output_norm=OutputNormSink(theirs, behind, 1e-5, 1.0, follow))
        close(mine, theirs, dtype)
        if follow is None:
            assert isinstance(got, ResidualCopy)
        else:
            assert isinstance(got, ReadyInput) and got.norm is following
            close(got.x, want.x, dtype)


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


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("nh,nkv,d,window,q_lens,kv_lens", [
    (4, 2, 64, 24, [1, 1, 1], [70, 1, 300]),             # single tokens
    (8, 1, 64, 1500, [1, 1], [5000, 2300]),              # single tokens behind keys that are split over workgroups and merged
    (4, 2, 64, 17, [9, 30, 2], [9, 155, 40]),            # short portions
    (8, 2, 64, 136, [600, 500], [600, 1500]),            # long portions
    (16, 4, 128, 100, [300], [900]),
    (20, 1, 32, 40, [1, 1, 40, 7], [800, 3, 100, 7]),    # more query heads to a key head than one tile of rows; single tokens before portions
    (3, 1, 272, 50, [1, 9, 30], [70, 9, 155]),           # beyond the tiled kernels
])
def test_a_loud_key_just_inside_and_just_outside_the_window_beside_a_silent_one(ops, dtype, nh, nkv, d, window, q_lens, kv_lens):
    """Every softmax has one more key of score 0 without a value.  The key that stands first in the last query's window is made
    loud, then the one before it: the first changes that query's result, the second does not, and both equal the reference."""
    ref, dt = TorchOps(), DTYPES[dtype]
    page = 16
    sinks = torch.zeros(nh).cuda()
    prefix = next((i for i, n in enumerate(q_lens) if n != 1), len(q_lens))
    longest = max(range(len(kv_lens)), key=lambda b: kv_lens[b])
    last_row = sum(q_lens[:longest + 1]) - 1
    results = {}
    for label, back in (("plain", None), ("inside", window - 1), ("outside", window)):
        q, k_cache, v_cache, tables, cu, lens = _paged_case(nh, nkv, d, q_lens, kv_lens, page, dt)
        if back is not None:
            place = kv_lens[longest] - 1 - back
            page_id, offset = int(tables[longest, place // page]), place % page
            for g in range(nkv):  # along the last query of the group's first head
                k_cache[page_id, g, offset] = 40.0 * torch.nn.functional.normalize(q[last_row].view(nh, d)[g * (nh // nkv)].float(), dim=0).to(dt)
            v_cache[page_id, :, :, offset] = 5.0
        args = (q, nh, nkv, d, k_cache, v_cache, page, tables, cu, lens, max(q_lens), max(kv_lens), 1.0 / math.sqrt(d), window, max(q_lens) == 1, Workspace(torch.device("cuda")))
        got = ops.paged_attention(*args, decode_prefix=prefix, sinks=sinks)
        close(got, ref.paged_attention(*args, sinks=sinks), dtype)
        results[label] = got[last_row].view(nh, d)[0].float()
    assert float((results["inside"] - results["plain"]).abs().max()) > 1.0
    assert torch.equal(results["outside"], results["plain"])


# ----------------------------------------------------------------------------------------------------
# the whole model
# ----------------------------------------------------------------------------------------------------
def rows_close(got, want, dtype, label, limit=0.08, share=0.9):
    if dtype == "float32":
        torch.testing.assert_close(got, want, msg=lambda m: f"{label}: {m}", **TOL[dtype])
    else:
        # bfloat16: rounding may send a token to another expert where two scores are close; such rows are few
        err = (got - want).abs().amax(-1) / want.abs().amax(-1).clamp(min=1.0)
        assert float((err < limit).float().mean()) >= share, f"{label}: {err}"


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
        if label in ("mixed", "recompute") and replayer.cache.groups:
            assert sum((len(t) + page - 1) // page for t in requests.values()) > replayer.cache.num_total_pages
    if dtype == "float32":
        for label in ("tail", "portions", "mixed", "recompute"):  # the ways of cutting agree with each other at least as closely
            for rid in requests:
                torch.testing.assert_close(results[label][rid], results["whole"][rid], rtol=1e-4, atol=3e-5)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("far_at,length", [(0, 600), (3, 200), (15, 200), (16, 200), (17, 200), (64, 200)])
def test_a_loud_token_far_back_in_the_states(tmp_path, dtype, far_at, length):
    """One early token is made loud and the states keep for long (decays near 1, removal rates and update gates near 0): hundreds of
    tokens on, far behind every window, the logits still depend on it and equal the plain model's, from a portion and from
    single tokens, written by one step and read by later ones, from a page's first or last place."""
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
    assert float(moved.median()) > 0.1
    requests = {"r0": tokens}
    cuts = (far_at + 1, 2, 100, 1, 3, 33, 2)
    for label, trace in (("whole", rc.whole(requests)), ("tail", rc.tail_one_by_one(requests, tail=40)), ("portions", rc.changing_portions(requests, sizes=cuts))):
        replayer = Replayer(folder, dtype, length + 16, block_size=16, max_live=2)
        got = rc.collect(trace, rc.run_trace(replayer, trace), requests)
        rows_close(got["r0"][-150:], right[-150:].float(), dtype, f"far {label}", limit=0.12, share=0.85)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_and_a_batch_against_each_request_alone(tmp_path, dtype):
    """A prompt of a few tokens, then 200 tokens one by one across many page borders; then four requests of unequal
    length decoded together, whose logits equal those of each request decoded alone."""
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
            np.testing.assert_allclose(row, alone[rid][k][0], rtol=1e-4 if dtype == "float32" else 8e-2, atol=2e-5 if dtype == "float32" else 8e-2)


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
        want = plain.forward(config, weights, tokens)[[0, 16, 29]].float().numpy()
        np.testing.assert_allclose(got, want, **(dict(rtol=2e-4, atol=3e-5) if dtype == "float32" else dict(rtol=8e-2, atol=8e-2)))
