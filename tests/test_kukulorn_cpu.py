"""Kukulorn on a CPU: the kernels' plain references stand in for the kernels; the configuration reader, the parts, the
loader, the cache manager with its state slots, the step function, replay, the scheduler and the entry point are the
product's.  The yardstick is ``plain_kukulorn`` (whole sequences, no cache, float64)."""
import copy
import json
import math

import pytest
import torch

import plain_kukulorn as plain
import replay_cases as rc
from helpers import Harness
from kukulorn_cases import CONFIGS, PAGE_SIZE, long_memory, prompts, random_weights, tensor_shapes, write_folder
from torch_ops import TorchOps
from velox_amd import Engine, EngineConfig, Request, SamplingParams
from velox_amd.cache.allocator import NULL_PAGE
from velox_amd.cache.manager import CacheManager
from velox_amd.config.model_config import ConfigError
from velox_amd.config.registry import config_from_dict, load_config
from velox_amd.engine.batch import StepEntry
from velox_amd.engine.engine import build_model
from velox_amd.engine.replay import Replayer
from velox_amd.parts import ModelSpec, PagedNeed, PartSpec, ScheduleEntry, kv_pages, make_part
from velox_amd.parts.base import NormedSum, SumOf
from velox_amd.weights import WeightsError, bind_from_checkpoint

TOL = dict(rtol=2e-4, atol=3e-5)


def close(got, want, msg=None):
    torch.testing.assert_close(got, want, msg=msg, rtol=2e-4, atol=3e-5 * max(1.0, float(want.abs().max())))


def logits_of(config, weights, tokens):
    return plain.forward(config, weights, tokens).float()


# ----------------------------------------------------------------------------------------------------------------------
# configuration and tensors
# ----------------------------------------------------------------------------------------------------------------------
def test_configuration_is_read_layer_by_layer_and_refused_where_it_cannot_run(tmp_path):
    config = config_from_dict(CONFIGS["A"])
    assert config.architecture == "Kukulorn" and config.width == 64 and config.loop == (1, 3, 3) and config.logit_softcap == 6.0
    model = build_model(config, torch.float32, "cpu", max_position=64)
    assert [e.layer for e in model.schedule] == [0, 1, 2, 1, 2, 1, 2, 3, 4]
    assert [i for i, e in enumerate(model.schedule) if e.begins_pass] == [1, 3, 5]
    assert {type(b).__name__ for b in model.blocks} == {"ParallelBlock"}
    full, pair, bare = (model.blocks[i].mixer for i in range(3))
    assert (full.num_heads, full.num_kv_heads, full.dim, full.vdim, full.cached_dim, full.conv_taps, full.scale) == (4, 2, 16, 12, 16, 3, 0.8)
    assert (full.softcap, full.gate, full.post_norm_eps, full.qkv_bias, full.out_bias, full.window) == (4.0, "channel", 1e-5, True, False, None)
    assert full.position.rotary_dim == 8 and full.position.bands == (4.0, 1.0, 4.0, 40.0) and bare.position.bands is None and bare.softcap == 2.5
    window, space = pair.mixers
    assert (window.window, window.keep_first, window.distance_bias, window.gate, window.qk_norm) == (7, 3, (10, 30.0), "head", "whole")
    assert window.qkv_bias and window.out_bias and window.cached_dim == 32
    assert (space.num_heads, space.groups, space.state, space.vdim, space.conv_taps, space.norm_groups, space.norm_eps) == (3, 1, 10, 12, 4, 2, 1e-5)
    assert pair.scales == (0.5, 0.5) and [n.prefix for n in pair.output_norms] == ["l1.mix.left.out", "l1.mix.right.out"]
    assert model.blocks[2].feed_forward.forward(None, None) is None and model.blocks[0].feed_forward.activation == "relu"
    needs = model.cache_needs()
    assert len(needs) == 9 and all(n is not None for n in needs)  # every pass has caches and states of its own
    assert needs[1].parts[0].window == 7 and needs[1].parts[0].keep_first == 3
    other = build_model(config_from_dict(CONFIGS["B"]), torch.float32, "cpu", max_position=32)
    assert other.pass_input is None and other.head.softcap is None and other.blocks[1].mixer.softcap is None
    assert other.blocks[0].mixer.mixers[0].keep_first == 0 and other.blocks[0].mixer.mixers[0].window == 11
    for change, message in (
        (lambda c: c["layers"][0].update(type="other"), "type"),
        (lambda c: c["layers"][0]["mlp"].update(kind="gated"), "kind"),
        (lambda c: c["layers"][0]["mixer"].update(heads=5), "multiple"),
        (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
        (lambda c: c["layers"][0]["mixer"].update(softcap=0.0, conv=-1), "conv"),
        (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "rot"),
        (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(high=1.0), "scaling"),
        (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(size=0), "mask"),
        (lambda c: c["layers"][1]["mixer"]["left"].pop("bias_max"), "bias_max"),
        (lambda c: c["layers"][1]["mixer"]["left"].pop("buckets"), "rel"),
        (lambda c: c["layers"][1]["mixer"]["right"].update(groups=2), "groups"),
        (lambda c: c["layers"][1]["mixer"]["right"].update(norm_groups=5), "norm_groups"),
        (lambda c: c["layers"][1]["mixer"].pop("right"), "right"),
        (lambda c: c["loop"].update(stop=6), "loop"),
        (lambda c: c["loop"].update(times=0), "loop"),
        (lambda c: c.update(logit_softcap=-1.0), "logit_softcap"),
        (lambda c: c.pop("width"), "width"),
    ):
        broken = copy.deepcopy(CONFIGS["A"])
        change(broken)
        with pytest.raises(ConfigError, match=message):
            config_from_dict(broken)
    folder = write_folder(tmp_path / "A", CONFIGS["A"], seed=1)  # (the rows of the bias tables come from the tensors' shapes)
    loaded = load_config(folder)
    assert "buckets" not in loaded.raw["layers"][1]["mixer"]["left"] and "tensor_shapes" not in loaded.to_json_dict()
    assert build_model(loaded, torch.float32, "cpu", max_position=32).blocks[3].mixer.mixers[0].distance_bias == (7, 14.0)


def test_every_tensor_is_named_and_shaped_as_the_design_says(tmp_path):
    for name, config in CONFIGS.items():
        folder = write_folder(tmp_path / name, config, seed=1)
        model = build_model(load_config(folder), torch.float32, "cpu", max_position=32)
        count = bind_from_checkpoint(model, folder, torch.float32, "cpu")
        assert count == sum(math.prod(s) for s in tensor_shapes(config).values()), name
    weights = random_weights(CONFIGS["A"], 1)
    weights["l0.mix.o.b"] = torch.ones(64)  # the full attention's output projection has no bias
    del weights["l1.mix.right.out"]
    folder = write_folder(tmp_path / "broken", CONFIGS["A"], seed=1, weights=weights)
    model = build_model(load_config(folder), torch.float32, "cpu", max_position=32)
    with pytest.raises(WeightsError) as caught:
        bind_from_checkpoint(model, folder, torch.float32, "cpu")
    assert caught.value.unexpected == ["l0.mix.o.b"] and caught.value.missing == ["l1.mix.right.out"]


def test_a_pass_needs_something_that_makes_its_input():
    layer = build_model(config_from_dict(CONFIGS["D"]), torch.float32, "cpu", max_position=8).spec.layers[0]
    spec = ModelSpec(vocab_size=8, hidden_size=48, max_position=8, layers=[layer], schedule=[ScheduleEntry(0, begins_pass=True)],
                     final_norm=PartSpec.of("rmsnorm", hidden_size=48, eps=1e-5))
    with pytest.raises(ValueError, match="pass_input"):
        spec.validate()


# ----------------------------------------------------------------------------------------------------------------------
# each mechanism alone: the framework's part, fed through the step's context and the cache manager, against the plain function
# ----------------------------------------------------------------------------------------------------------------------
def _harness(tmp_path, name, seed=2, weights=None):
    folder = write_folder(tmp_path / name, CONFIGS[name], seed=seed, weights=weights)
    config, tensors = plain.read_folder(folder)
    return Harness(folder, TorchOps(), torch.float32, "cpu", PAGE_SIZE[name], 64, max_num_seqs=3, max_num_tokens=128), config, tensors


def _whole(value):
    """A mixer's output as a tensor (a sum whose terms still have norms to pass is worked out)."""
    return TorchOps._one_delta(value)


def _mixer_in_portions(harness, entry, x, cuts):
    """Runs schedule entry ``entry``'s mixer alone on rows ``x`` of one sequence, cut into portions."""
    seq = harness.cache.new_sequence()
    block = harness.model.blocks[harness.model.schedule[entry].layer]
    out, at = [], 0
    for n in cuts:
        assert harness.cache.append(seq, at, n)
        ctx = harness.runner.builder.build([StepEntry(seq, [0] * n, at, [])], harness.runner.ops, torch.float32, harness.runner.workspace)
        out.append(_whole(block.mixer.forward(x[at:at + n].contiguous(), ctx, ctx.cache_view(entry), True)))
        at += n
        harness.cache.release_behind_window(seq, at)
    harness.cache.free_sequence(seq)
    return torch.cat(out)


@pytest.mark.parametrize("name,entry", [("A", 0), ("A", 1), ("A", 2), ("A", 4), ("A", 7), ("A", 8), ("B", 0), ("B", 1), ("B", 2), ("D", 0), ("D", 1), ("E", 1), ("E", 2)])
def test_each_mixer_alone_whole_and_in_portions(tmp_path, name, entry):
    harness, config, weights = _harness(tmp_path, name)
    index = plain.run_order(config)[entry][0]
    layer = config["layers"][index]
    x = torch.randn(29, config["width"])
    want = plain.MIXERS[layer["type"]](x.double(), weights, f"l{index}.mix.", layer["mixer"], config["norm"]["eps"]).float()
    assert float(want.abs().max()) > 0.1
    for cuts in ((29,), (1,) * 29, (5, 2, 1, 9, 2, 10), (2, 27)):
        got = _mixer_in_portions(harness, entry, x, cuts)
        torch.testing.assert_close(got, want, msg=lambda m: f"{name} run {entry} cut {cuts}: {m}", **TOL)


@pytest.mark.parametrize("name,side", [("A", 0), ("A", 1), ("B", 0), ("B", 1), ("D", 0), ("D", 1), ("E", 0)])
def test_each_side_of_a_pair_alone(tmp_path, name, side):
    harness, config, weights = _harness(tmp_path, name)
    index = next(i for i, e in enumerate(config["layers"]) if e["type"] == "parallel")
    entry = [layer for layer, _ in plain.run_order(config)].index(index)
    x = torch.randn(21, config["width"])
    function, below = ((plain.kept_window_attention, "left"), (plain.state_space_mixer, "right"))[side]
    want = function(x.double(), weights, f"l{index}.mix.{below}.", config["layers"][index]["mixer"][below], config["norm"]["eps"]).float()
    mixer = harness.model.blocks[index].mixer.mixers[side]
    for cuts in ((21,), (1,) * 21, (2, 5, 1, 13)):
        seq = harness.cache.new_sequence()
        rows, at = [], 0
        for n in cuts:
            assert harness.cache.append(seq, at, n)
            ctx = harness.runner.builder.build([StepEntry(seq, [0] * n, at, [])], harness.runner.ops, torch.float32, harness.runner.workspace)
            rows.append(mixer.forward(x[at:at + n].contiguous(), ctx, ctx.cache_view(entry).views[side]))
            at += n
            harness.cache.release_behind_window(seq, at)
        harness.cache.free_sequence(seq)
        torch.testing.assert_close(torch.cat(rows), want, msg=lambda m: f"{name} {below} cut {cuts}: {m}", **TOL)


def test_feed_forward_alone(tmp_path):
    harness, config, weights = _harness(tmp_path, "A")
    x = torch.randn(11, config["width"])
    want = plain.feed_forward(x.double(), weights, "l1.mlp.").float()
    assert float(want.abs().max()) > 0.1
    seq = harness.cache.new_sequence()
    assert harness.cache.append(seq, 0, 11)
    ctx = harness.runner.builder.build([StepEntry(seq, [0] * 11, 0, [])], harness.runner.ops, torch.float32, harness.runner.workspace)
    torch.testing.assert_close(harness.model.blocks[1].feed_forward.forward(x, ctx), want, **TOL)


def test_norms_behind_side_by_side_mixers_and_the_rows_joined_before_a_pass():
    """A sum whose terms have norms of their own, in all the forms its terms travel in; chosen rows change nothing; the pass's
    input is made of the residual with everything that is pending, and clears it."""
    class Ctx:
        ops = TorchOps()
        dtype = torch.float32

    norm = make_part("norm", "rmsnorm", prefix="", hidden_size=10, eps=1e-3, weight_name="")
    norm.weight = 1.0 + 0.2 * torch.randn(10)
    weights = (1.0 + 0.2 * torch.randn(10), 1.0 + 0.2 * torch.randn(10))
    x, a, b, p = torch.randn(7, 10), torch.randn(2, 7, 10), torch.randn(7, 10), torch.randn(3, 7, 10)
    normed = 0.5 * (plain.rms_norm(a.double().sum(0), weights[0].double(), 1e-2) + plain.rms_norm(b.double(), weights[1].double(), 1e-2))
    for plain_term in (p, p.sum(0), None):
        delta = NormedSum((a, b), weights, (0.5, 0.5), 1e-2, plain_term)
        want_x = x.double() + normed + (0.0 if plain_term is None else p.double().sum(0))
        want = plain.rms_norm(want_x, norm.weight.double(), 1e-3).float()
        residual, rows = x.clone(), torch.tensor([6, 0, 3], dtype=torch.int32)
        torch.testing.assert_close(norm.forward(residual, delta, Ctx, rows=rows), want[rows.long()], **TOL)
        assert torch.equal(residual, x)
        torch.testing.assert_close(norm.forward(residual, delta, Ctx), want, **TOL)
        torch.testing.assert_close(residual, want_x.float(), **TOL)
        joint = make_part("pass_input", "linear", hidden_size=10, name="in")
        joint.weight = torch.randn(10, 20)
        start, residual = torch.randn(7, 10), x.clone()
        pending = joint.forward(residual, delta, start, Ctx)
        torch.testing.assert_close(residual + pending, (torch.cat([want_x, start.double()], -1) @ joint.weight.double().T).float(), **TOL)
        assert not residual.any()
    residual = x.clone()
    pending = joint.forward(residual, SumOf(p, b), start, Ctx)
    torch.testing.assert_close(pending, (torch.cat([x.double() + p.double().sum(0) + b.double(), start.double()], -1) @ joint.weight.double().T).float(), **TOL)


@pytest.mark.parametrize("dims,base,bands", [(16, 10000.0, (8.0, 1.0, 4.0, 512.0)), (32, 250.0, (3.0, 0.5, 2.0, 40.0)), (8, 100.0, (4.0, 1.0, 4.0, 40.0))])
def test_frequencies_are_stretched_by_wavelength(dims, base, bands):
    """The tables at every position against the plain frequencies; some stay, some are divided, some lie between."""
    position = make_part("position", "rotary", rotary_dim=dims, theta=base, max_position=700, exact_angles=True, bands=bands)
    position.finalize(torch.device("cpu"), torch.float32)
    scaling = dict(zip(("factor", "low", "high", "original"), bands))
    freq = torch.tensor(plain.banded_frequencies(dims, base, scaling), dtype=torch.float64)
    bare = torch.tensor(plain.banded_frequencies(dims, base, None), dtype=torch.float64)
    ratio = freq / bare
    assert bool((ratio == 1).any()) and bool((ratio - 1 / bands[0]).abs().min() < 1e-12) and bool(((ratio < 0.99) & (ratio > 1.01 / bands[0])).any())
    angles = torch.outer(torch.arange(700, dtype=torch.float64), freq)
    torch.testing.assert_close(position.cos, angles.cos().float(), rtol=0, atol=1e-6)
    torch.testing.assert_close(position.sin, angles.sin().float(), rtol=0, atol=1e-6)
    for wrong in ((4.0, 2.0, 2.0, 40.0), (0.0, 1.0, 2.0, 40.0)):
        with pytest.raises(ValueError):
            make_part("position", "rotary", rotary_dim=8, theta=10.0, max_position=8, exact_angles=True, bands=wrong)


@pytest.mark.parametrize("window,keep", [(5, 3), (5, 4), (5, 5), (4, 13), (9, 1)])
def test_pages_of_kept_tokens_stay_and_those_between_go_back(window, keep):
    """Page by page, while a request grows one token at a time: exactly the pages that hold a token a later query can see are
    held, whatever lay in them before."""
    page = 4
    manager = CacheManager([kv_pages(1, 16, window, keep)], page, 32, 2, torch.float32, "cpu")
    other, seq = manager.new_sequence(), manager.new_sequence()
    assert manager.append(other, 0, 9)
    for n in range(70):
        assert manager.append(seq, n, 1)
        manager.release_behind_window(seq, n + 1)
        visible = set(plain.visible(n + 1, window, keep))  # what the next query sees of what is there
        held = {j // page for j in visible if j <= n}
        table = seq.tables[0]
        assert {i for i, p in enumerate(table) if p != NULL_PAGE} == held | {i for i in range(len(table)) if i * page > n + 1 - window}, n
        manager.assert_consistent([other, seq])
    manager.free_sequence(seq)
    manager.free_sequence(other)
    assert manager.num_used_pages() == 0
    assert kv_pages(1, 16, None, 7).keep_first == 0
    with pytest.raises(ValueError):
        PagedNeed((("k", (-1, 4), None),), 5, -1)


def test_layer_outputs_one_by_one(tmp_path):
    """The residual stream after every layer run, from the framework's blocks run one at a time, against the plain model's."""
    for name in ("A", "E"):
        harness, config, weights = _harness(tmp_path, name, seed=5)
        tokens = prompts(config["vocab"], [23], seed=8)["r0"]
        want = []
        plain.forward(config, weights, tokens, want)
        seq = harness.cache.new_sequence()
        assert harness.cache.append(seq, 0, len(tokens))
        ctx = harness.runner.builder.build([StepEntry(seq, tokens, 0, [])], harness.runner.ops, torch.float32, harness.runner.workspace)
        model = harness.model
        residual, pending = model.begin(ctx.token_ids, ctx), None
        for index in range(len(model.schedule)):
            pending = model.run_schedule(residual, pending, ctx, first=index, last=index + 1)
            scratch = residual.clone()
            model.final_norm.forward(scratch, pending, ctx)  # (works in what the layer's sub-layers left pending)
            torch.testing.assert_close(scratch, want[index].float(), msg=lambda m: f"{name} after layer run {index}: {m}",
                                       rtol=2e-4, atol=3e-5 * max(1.0, float(want[index].abs().max())))
        harness.cache.free_sequence(seq)


# ----------------------------------------------------------------------------------------------------------------------
# whole models: every way of cutting, batches, pages and slots that are used again
# ----------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("name", ["A", "B", "D", "E"])
def test_all_ways_of_cutting_agree_with_the_plain_model(tmp_path, name):
    """Whole prompts; the last tokens one by one (more of them than a window reaches back); portions of 1 to 16 tokens (many
    of two); up to four requests mixed in a pool so small that pages are used again, with seven requests on four state slots;
    requests that are ended half way and recomputed in slots that others have used since."""
    folder = write_folder(tmp_path / name, CONFIGS[name], seed=2)
    config, weights = plain.read_folder(folder)
    requests = prompts(config["vocab"], [41, 1, 17, 58, 9, 33, 2], seed=3)
    expected = {rid: logits_of(config, weights, tokens) for rid, tokens in requests.items()}
    assert all(float(e.abs().max()) > 1.0 for e in expected.values())  # logits of order one and more: the tolerances bite
    page = PAGE_SIZE[name]
    for label, trace in (("whole", rc.whole(requests)), ("tail", rc.tail_one_by_one(requests, tail=30)),
                         ("portions", rc.changing_portions(requests)), ("mixed", rc.mixed(requests, seed=5)),
                         ("recompute", rc.mixed(requests, seed=6, preempt=("r0", "r3")))):
        replayer = Replayer(folder, "float32", rc.tokens_needed(trace, page), block_size=page, device="cpu", ops=TorchOps(), max_live=4)
        outputs = rc.run_trace(replayer, trace)
        got = rc.collect(trace, outputs, requests)
        for rid in requests:
            close(got[rid], expected[rid], msg=lambda m: f"{name} {label} {rid}: {m}")
        if label in ("mixed", "recompute"):
            assert sum((len(t) + page - 1) // page for t in requests.values()) > replayer.cache.num_total_pages


def test_a_left_out_mechanism_would_show(monkeypatch):
    """The weights are sharp enough that the tests above can fail: each mechanism, taken out of the plain model or moved by
    one, changes the logits far beyond the tolerance."""
    config = CONFIGS["A"]
    weights = {k: v.double() for k, v in random_weights(config, 2).items()}
    tokens = prompts(config["vocab"], [40], seed=4)["r0"]
    right = plain.forward(config, weights, tokens)

    def moved(change_config=None, change_weights=None, **patched):
        c, w = json.loads(json.dumps(config)), dict(weights)
        if change_config:
            change_config(c)
        if change_weights:
            change_weights(w)
        with monkeypatch.context() as patch:
            for name, value in patched.items():
                patch.setattr(plain, name, value)
            return float((right - plain.forward(c, w, tokens))[-8:].abs().max())

    pair = lambda c: c["layers"][1]["mixer"]  # noqa: E731
    for size in (6, 8):
        assert moved(lambda c: pair(c)["left"]["mask"].update(size=size)) > 0.02, size
    for keep in (0, 2, 4):
        assert moved(lambda c: pair(c)["left"]["mask"].update(keep_first=keep)) > 0.02, keep
    assert moved(lambda c: pair(c)["left"].pop("mask")) > 0.05
    assert moved(lambda c: pair(c)["left"].update(bias_max=25.0)) > 0.005 and moved(lambda c: pair(c)["left"].update(scale=0.8)) > 0.02
    assert moved(lambda c: c["layers"][3]["mixer"]["left"].update(bias_max=9.0)) > 0.005
    assert moved(lambda c: pair(c)["right"].update(norm_groups=1)) > 0.005
    assert moved(lambda c: c["layers"][0]["mixer"].pop("softcap")) > 0.02 and moved(lambda c: c["layers"][2]["mixer"].update(softcap=2.4)) > 0.002
    assert moved(lambda c: c["layers"][0]["mixer"]["rot"].pop("scaling")) > 0.02 and moved(lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=3.0)) > 0.005
    assert moved(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=6)) > 0.02 and moved(lambda c: c["layers"][2]["mixer"].update(scale=0.55)) > 0.02
    assert moved(lambda c: c["loop"].update(times=2)) > 0.05 and moved(lambda c: c["loop"].update(stop=2)) > 0.05 and moved(lambda c: c["loop"].update(start=2)) > 0.05
    assert moved(lambda c: c.pop("loop")) > 0.05 and moved(lambda c: c.pop("logit_softcap")) > 0.05
    assert moved(rotate_halves=lambda x, dims, base, scaling: x) > 0.05
    assert moved(causal_conv=lambda u, w: u * w[:, -1]) > 0.05
    assert moved(silu=lambda z: torch.relu(z)) > 0.05
    assert moved(distance_bucket=lambda n, b, far: min(n, b - 1)) > 0.02
    assert moved(gated_group_norm=lambda y, z, w, g, eps: plain.over_rms(y.reshape(y.shape[0], g, -1), eps).reshape(y.shape) * w * plain.silu(z)) > 0.02
    assert moved(state_space_scan=lambda x, b, c, step, rate, skip: skip[None, :, None] * x) > 0.02
    for name in ("loop.in", "l0.mix.q.b", "l0.mix.v.conv", "l0.mix.g", "l1.mix.left.o.b", "l1.mix.left.q.norm", "l1.mix.left.rel", "l1.mix.left.g", "l1.mix.right.conv.b",
                 "l1.mix.right.dt_bias", "l1.mix.right.A_log", "l1.mix.right.D", "l1.mix.right.norm", "l1.mix.left.out", "l1.mix.right.out", "l1.norm1"):
        assert moved(change_weights=lambda w: w.update({name: w[name].flip(0)})) > 0.005, name
    shifted = plain.forward(config, weights, tokens[1:])  # one token less: states, windows, kept tokens and positions all differ
    assert float((right[-1] - shifted[-1]).abs().max()) > 0.02


@pytest.mark.parametrize("name,cuts", [("E", (200,)), ("E", (3, 1, 192, 2, 1, 1)), ("E", (12, 1, 183) + (1,) * 4), ("A", (16, 15, 1, 66, 2) + (1,) * 10)])
def test_what_loud_first_tokens_wrote_is_read_far_later(tmp_path, name, cuts):
    """A state that is dropped or a kept page that is given back loses the first tokens: prompts that differ in one of them only
    give different logits at their end, and the framework agrees with the plain model on each, however the prompt is cut."""
    config = CONFIGS[name]
    weights = long_memory(random_weights(config, 4))
    folder = write_folder(tmp_path / name, config, seed=4, weights=weights)
    config, tensors = plain.read_folder(folder)
    n = sum(cuts)
    base = prompts(config["vocab"], [n], seed=9)["r0"]
    texts = {"base": base}
    for place in (0, 2, 12, 13):
        texts[f"other{place}"] = base[:place] + [(base[place] + 1) % config["vocab"]] + base[place + 1:]
    want = {rid: logits_of(config, tensors, toks)[-4:] for rid, toks in texts.items()}
    for rid in texts:
        assert rid == "base" or float((want["base"] - want[rid]).abs().max()) > 2e-3, rid  # the far token shows
    page = PAGE_SIZE[name]
    for rid, toks in texts.items():
        replayer = Replayer(folder, "float32", (n + page - 1) // page * page, block_size=page, device="cpu", ops=TorchOps(), max_live=2)
        at, rows = 0, []
        for i, c in enumerate(cuts):
            out = replayer.step({"step": i, "entries": [{"id": rid, "tokens": toks[at:at + c], "want": list(range(c))}], "end": [rid] if at + c == n else []})
            rows.append(torch.from_numpy(out))
            at += c
        close(torch.cat(rows)[-4:], want[rid], msg=lambda m: f"{name} {cuts} {rid}: {m}")


def test_a_slot_that_is_used_again_starts_from_nothing(tmp_path):
    """One state slot: every request starts in the slot the one before it left, and must not see what it wrote there; a
    request that comes again gives the same logits again."""
    folder = write_folder(tmp_path / "A", CONFIGS["A"], seed=2)
    config, weights = plain.read_folder(folder)
    requests = prompts(config["vocab"], [19, 3, 1, 26], seed=11)
    replayer = Replayer(folder, "float32", 32, block_size=4, device="cpu", ops=TorchOps(), max_live=1)
    for turn in range(2):
        for rid, toks in requests.items():
            half = max(1, len(toks) // 2)
            first = replayer.step({"step": 0, "entries": [{"id": rid, "tokens": toks[:half], "want": list(range(half))}], "end": [] if half < len(toks) else [rid]})
            rows = [torch.from_numpy(first)]
            if half < len(toks):
                rows.append(torch.from_numpy(replayer.step({"step": 1, "entries": [{"id": rid, "tokens": toks[half:], "want": list(range(len(toks) - half))}], "end": [rid]})))
            close(torch.cat(rows), logits_of(config, weights, toks), msg=lambda m: f"turn {turn} {rid}: {m}")
            assert replayer.cache.state.num_free == 1 and replayer.cache.num_used_pages() == 0


def test_long_decoding_past_every_window(tmp_path):
    """A prompt shorter than the kept tokens and then 120 tokens one by one: the windows pass over decoded tokens only, pages
    between the kept ones and the window go back to the pool, the states are carried 120 times."""
    for name in ("A", "E"):
        folder = write_folder(tmp_path / name, CONFIGS[name], seed=6)
        config, weights = plain.read_folder(folder)
        toks = prompts(config["vocab"], [122], seed=12)["r0"]
        want = logits_of(config, weights, toks)
        replayer = Replayer(folder, "float32", 124, block_size=4, device="cpu", ops=TorchOps(), max_live=1)
        rows = [torch.from_numpy(replayer.step({"step": 0, "entries": [{"id": "a", "tokens": toks[:2], "want": [0, 1]}], "end": []}))]
        for i in range(2, 122):
            rows.append(torch.from_numpy(replayer.step({"step": i, "entries": [{"id": "a", "tokens": [toks[i]], "want": [0]}], "end": ["a"] if i == 121 else []})))
        close(torch.cat(rows), want)


# ----------------------------------------------------------------------------------------------------------------------
# the entry point
# ----------------------------------------------------------------------------------------------------------------------
def plain_greedy(config, weights, prompt, n):
    tokens = list(prompt)
    for _ in range(n):
        tokens.append(int(plain.forward(config, weights, tokens)[-1].argmax()))
    return tokens[len(prompt):]


@pytest.mark.parametrize("name", ["A", "E"])
def test_greedy_generation_through_the_entry_point_with_preemption(tmp_path, name):
    """The scheduler, the step function and the sampler around the model: greedy tokens equal the plain model's, together and
    alone, in portions of seven tokens, also when the pool is so small that requests are preempted and computed again.
    Prefixes are not shared: a state of fixed size stands for tokens that a sharer would skip."""
    folder = write_folder(tmp_path / name, CONFIGS[name], seed=2)
    config, weights = plain.read_folder(folder)
    texts = list(prompts(config["vocab"], [5, 19, 13, 26], seed=7).values())
    want = [plain_greedy(config, weights, p, 8) for p in texts]

    def engine_for(**overrides):
        options = dict(model=folder, dtype="float32", device="cpu", max_model_len=96, max_num_seqs=4, max_num_batched_tokens=32,
                       max_prefill_chunk_size=7, block_size=4, num_gpu_blocks=96, enable_cuda_graphs=False, seed=0)
        options.update(overrides)
        return Engine.from_pretrained(EngineConfig(**options), ops=TorchOps())

    def requests(prefix):
        return [Request(f"{prefix}{i}", p, SamplingParams(temperature=0.0, max_tokens=8, ignore_eos=True)) for i, p in enumerate(texts)]

    engine = engine_for()
    assert engine.cache.prefix is None
    assert [r.output_token_ids for r in engine.generate(requests("a"))] == want
    assert [r.output_token_ids for r in engine.generate(requests("again"))] == want  # in slots and pages that the first ones used
    alone = engine.generate([Request("alone", texts[1], SamplingParams(temperature=0.0, max_tokens=8, ignore_eos=True))])[0]
    assert alone.output_token_ids == want[1]
    two_slots = engine_for(max_num_seqs=2)
    assert [r.output_token_ids for r in two_slots.generate(requests("s"))] == want
    tight = engine_for(num_gpu_blocks=11)
    assert [r.output_token_ids for r in tight.generate(requests("t"))] == want
    assert tight.cache.num_used_pages() == 0
    tight.cache.assert_consistent([])
