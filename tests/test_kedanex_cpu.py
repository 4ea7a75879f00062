"""Kedanex on a CPU: the kernels' plain references stand in for the kernels; the configuration reader, the parts, the
loader, the cache manager with its state slots, the step function, replay, the scheduler and the entry point are the
product's.  The yardstick is ``plain_kedanex`` (whole sequences, no cache, float64)."""
import copy
import json
import math

import pytest
import torch

import plain_kedanex as plain
import replay_cases as rc
from helpers import Harness
from kedanex_cases import CONFIGS, PAGE_SIZE, long_memory, prompts, random_weights, tensor_shapes, write_folder
from torch_ops import TorchOps
from velox_amd import Engine, EngineConfig, Request, SamplingParams
from velox_amd.config.model_config import ConfigError
from velox_amd.config.registry import config_from_dict, load_config
from velox_amd.engine.batch import StepEntry
from velox_amd.engine.engine import build_model
from velox_amd.engine.replay import Replayer
from velox_amd.parts.base import NormedDelta, ReadyInput
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
    assert config.architecture == "Kedanex" and config.width == 64 and len(config.layers) == 8
    model = build_model(config, torch.float32, "cpu", max_position=64)
    assert len(model.blocks) == 5 and [e.layer for e in model.schedule] == [0, 1, 2, 3, 4, 2, 1, 3]  # three layers run earlier ones' weights
    assert {type(b).__name__ for b in model.blocks} == {"SandwichBlock"}
    delta, gru, window = (model.blocks[i].mixer for i in range(3))
    assert (delta.num_heads, delta.dim, delta.vdim, delta.decay_rank) == (3, 12, 12, 5) and abs(delta.decay_scale - math.exp(-0.5)) < 1e-12
    assert (gru.width, gru.shift) == (20, 0.5)
    assert (window.num_heads, window.num_kv_heads, window.dim, window.cached_dim, window.window, window.scale) == (4, 2, 16, 16, 6, 0.7)
    assert window.values_are_keys and window.sink_score == 0.0 and window.post_norm_eps == 1e-5 and not window.qkv_bias and not window.out_bias
    assert window.position.rotary_dim == 8 and window.position.theta == 100.0 and window.position.layout == "halves"
    mlp, routed = model.blocks[0].feed_forward, model.blocks[1].feed_forward
    assert mlp.activation == "poly_norm" and mlp.intermediate_size == 40 and mlp.norm_eps == 1e-5
    assert (routed.num_experts, routed.top, routed.score, routed.renormalize, routed.scale_input) == (6, 2, "softmax", True, False)
    assert not model.blocks[3].has_feed_forward
    needs = model.cache_needs()
    assert len(needs) == 8 and all(n is not None for n in needs)  # every run of a layer has a cache or state of its own
    assert needs[0].tensors == (("state", (3, 12, 12), torch.float32),) and needs[1].tensors == (("state", (20,), torch.float32),) and needs[2].window == 6
    other = build_model(config_from_dict(CONFIGS["B"]), torch.float32, "cpu", max_position=32)
    assert other.blocks[0].mixer.window is None and other.blocks[0].mixer.position is None
    for change, message in (
        (lambda c: c["layers"][0].update(type="other"), "type"),
        (lambda c: c["layers"][0]["mlp"].update(kind="gated"), "kind"),
        (lambda c: c["layers"][1]["mlp"]["router"].update(top=7), "top"),
        (lambda c: c["layers"][2]["mixer"].update(heads=5), "multiple"),
        (lambda c: c["layers"][2]["mixer"].update(vdim=8), "vdim"),
        (lambda c: c["layers"][2]["mixer"]["mask"].update(size=0), "mask.size"),
        (lambda c: c["layers"][2]["mixer"]["rot"].update(dims=18), "rot"),
        (lambda c: c["layers"][2]["mixer"].pop("scale"), "scale"),
        (lambda c: c["layers"][1]["mixer"].update(width=0), "width"),
        (lambda c: c["layers"][5].update(weights_of=5), "weights_of"),
        (lambda c: c["layers"][5].update(weights_of=1), "type"),
        (lambda c: c["layers"][0]["mixer"].pop("w1_rank"), "w1"),
        (lambda c: c.pop("width"), "width"),
    ):
        broken = copy.deepcopy(CONFIGS["A"])
        change(broken)
        with pytest.raises(ConfigError, match=message):
            config_from_dict(broken)
    folder = write_folder(tmp_path / "A", CONFIGS["A"], seed=1)  # (the inner sizes of the low-rank maps come from the tensors' shapes)
    loaded = load_config(folder)
    assert "w1_rank" not in loaded.raw["layers"][0]["mixer"] and "tensor_shapes" not in loaded.to_json_dict()
    assert build_model(loaded, torch.float32, "cpu", max_position=32).blocks[3].mixer.decay_rank == 7


def test_a_layer_may_run_a_later_layers_weights():
    """The owner may stand behind the layer that runs its weights, or be reached over another layer that owns none."""
    config = copy.deepcopy(CONFIGS["E"])
    config["layers"][0]["weights_of"] = 2
    del config["layers"][2]["weights_of"]
    model = build_model(config_from_dict(config), torch.float32, "cpu", max_position=32)
    assert [e.layer for e in model.schedule] == [1, 0, 1] and model.blocks[1].prefix == "l2."


def test_every_tensor_is_named_and_shaped_as_the_design_says(tmp_path):
    for name, config in CONFIGS.items():
        folder = write_folder(tmp_path / name, config, seed=1)
        model = build_model(load_config(folder), torch.float32, "cpu", max_position=32)
        count = bind_from_checkpoint(model, folder, torch.float32, "cpu")
        assert count == sum(math.prod(s) for s in tensor_shapes(config).values()), name
    weights = random_weights(CONFIGS["A"], 1)
    weights["l3.norm2b"] = torch.ones(64)  # a layer without a feed-forward has neither of its norms
    del weights["l2.norm1b"]
    folder = write_folder(tmp_path / "broken", CONFIGS["A"], seed=1, weights=weights)
    model = build_model(load_config(folder), torch.float32, "cpu", max_position=32)
    with pytest.raises(WeightsError) as caught:
        bind_from_checkpoint(model, folder, torch.float32, "cpu")
    assert caught.value.unexpected == ["l3.norm2b"] and caught.value.missing == ["l2.norm1b"]


# ----------------------------------------------------------------------------------------------------------------------
# each mechanism alone: the framework's part, fed through the step's context and the cache manager, against the plain function
# ----------------------------------------------------------------------------------------------------------------------
def _harness(tmp_path, name, seed=2, weights=None):
    folder = write_folder(tmp_path / name, CONFIGS[name], seed=seed, weights=weights)
    config, tensors = plain.read_folder(folder)
    return Harness(folder, TorchOps(), torch.float32, "cpu", PAGE_SIZE[name], 64, max_num_seqs=3, max_num_tokens=128), config, tensors


def _mixer_in_portions(harness, entry, x, cuts):
    """Runs schedule entry ``entry``'s mixer alone on rows ``x`` of one sequence, cut into portions."""
    seq = harness.cache.new_sequence()
    block = harness.model.blocks[harness.model.schedule[entry].layer]
    out, at = [], 0
    for n in cuts:
        assert harness.cache.append(seq, at, n)
        ctx = harness.runner.builder.build([StepEntry(seq, [0] * n, at, [])], harness.runner.ops, torch.float32, harness.runner.workspace)
        out.append(block.mixer.forward(x[at:at + n].contiguous(), ctx, ctx.cache_view(entry), True))
        at += n
        harness.cache.release_behind_window(seq, at)
    harness.cache.free_sequence(seq)
    return torch.cat(out)


@pytest.mark.parametrize("name,entry", [(n, e) for n in ("A", "B", "D") for e in range(3)] + [("A", 4), ("B", 3)])
def test_each_mixer_alone_whole_and_in_portions(tmp_path, name, entry):
    harness, config, weights = _harness(tmp_path, name)
    layer = config["layers"][entry]
    x = torch.randn(29, config["width"])
    want = plain.MIXERS[layer["type"]](x.double(), weights, f"l{entry}.mix.", layer["mixer"], config["norm"]["eps"]).float()
    assert float(want.abs().max()) > 0.1
    for cuts in ((29,), (1,) * 29, (5, 2, 1, 9, 2, 10), (2, 27)):
        got = _mixer_in_portions(harness, entry, x, cuts)
        torch.testing.assert_close(got, want, msg=lambda m: f"{name} layer {entry} cut {cuts}: {m}", **TOL)


@pytest.mark.parametrize("name,entry", [("A", 0), ("A", 1), ("A", 2), ("A", 4), ("B", 1), ("B", 2), ("D", 0)])
def test_each_feed_forward_alone(tmp_path, name, entry):
    harness, config, weights = _harness(tmp_path, name)
    x = torch.randn(11, config["width"])
    want = plain.feed_forward(config["layers"][entry]["mlp"], x.double(), weights, f"l{entry}.mlp.", config["norm"]["eps"]).float()
    assert float(want.abs().max()) > 0.1
    seq = harness.cache.new_sequence()
    assert harness.cache.append(seq, 0, 11)
    ctx = harness.runner.builder.build([StepEntry(seq, [0] * 11, 0, [])], harness.runner.ops, torch.float32, harness.runner.workspace)
    torch.testing.assert_close(harness.model.blocks[entry].feed_forward.forward(x, ctx), want, **TOL)


def test_norms_behind_and_before_a_sub_layer():
    """A delta with a norm of its own, in all the forms it travels in; chosen rows change nothing; a ready input goes to
    its norm only."""
    from velox_amd.parts import make_part

    class Ctx:
        ops = TorchOps()
        dtype = torch.float32

    inner, outer = (make_part("norm", "rmsnorm", prefix="", hidden_size=10, eps=1e-3, weight_name="") for _ in range(2))
    inner.weight, outer.weight = 1.0 + 0.2 * torch.randn(10), 1.0 + 0.2 * torch.randn(10)
    x, y = torch.randn(7, 10), torch.randn(2, 7, 10)
    want_x = x.double() + plain.rms_norm(y.double().sum(0), inner.weight.double(), 1e-3)
    want = plain.rms_norm(want_x, outer.weight.double(), 1e-3).float()
    for delta in (y, y.sum(0)):
        residual = x.clone()
        rows = torch.tensor([6, 0, 3], dtype=torch.int32)
        torch.testing.assert_close(outer.forward(residual, NormedDelta(delta, inner), Ctx, rows=rows), want[rows.long()], **TOL)
        assert torch.equal(residual, x)
        torch.testing.assert_close(outer.forward(residual, NormedDelta(delta, inner), Ctx), want, **TOL)
        torch.testing.assert_close(residual, want_x.float(), **TOL)
    assert outer.forward(x, ReadyInput(y[0], outer), Ctx) is not None
    with pytest.raises(ValueError):
        inner.forward(x, ReadyInput(y[0], outer), Ctx)


def test_layer_outputs_one_by_one(tmp_path):
    """The residual stream after every layer run, from the framework's blocks run one at a time, against the plain model's."""
    harness, config, weights = _harness(tmp_path, "A", seed=5)
    tokens = prompts(config["vocab"], [23], seed=8)["r0"]
    want = []
    plain.forward(config, weights, tokens, want)
    seq = harness.cache.new_sequence()
    assert harness.cache.append(seq, 0, len(tokens))
    ctx = harness.runner.builder.build([StepEntry(seq, tokens, 0, [])], harness.runner.ops, torch.float32, harness.runner.workspace)
    model = harness.model
    residual, pending = model.embed(ctx.token_ids, ctx), None
    for index in range(len(model.schedule)):
        pending = model.run_schedule(residual, pending, ctx, first=index, last=index + 1)
        scratch = residual.clone()
        if not isinstance(pending, ReadyInput):  # (the experts' last kernel has worked everything in already)
            model.final_norm.forward(scratch, pending, ctx)  # (works in what the layer's last sub-layer left pending)
        torch.testing.assert_close(scratch, want[index].float(), msg=lambda m: f"after layer run {index}: {m}",
                                   rtol=2e-4, atol=3e-5 * max(1.0, float(want[index].abs().max())))


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
        if label in ("mixed", "recompute") and replayer.cache.groups:
            assert sum((len(t) + page - 1) // page for t in requests.values()) > replayer.cache.num_total_pages


def test_a_left_out_mechanism_would_show(monkeypatch):
    """The weights are sharp enough that the tests above can fail: each mechanism, taken out of the plain model or moved by
    one, changes the logits far beyond the tolerance."""
    config = CONFIGS["A"]
    weights = {k: v.double() for k, v in random_weights(config, 2).items()}
    tokens = prompts(config["vocab"], [40], seed=4)["r0"]
    right = plain.forward(config, weights, tokens)

    def moved(change_config=None, change_weights=None, **patched):
        c, w = json.loads(json.dumps(config)), dict(weights)  # (entries that share a mixer come apart)
        if change_config:
            change_config(c)
        if change_weights:
            change_weights(w)
        with monkeypatch.context() as patch:
            for name, value in patched.items():
                patch.setattr(plain, name, value)
            return float((right - plain.forward(c, w, tokens))[-8:].abs().max())

    attend = lambda c: c["layers"][2]["mixer"]  # noqa: E731  (layer 5 repeats its entry and follows it)

    def both(change):
        def apply(c):
            change(c["layers"][2]["mixer"])
            change(c["layers"][5]["mixer"])
        return apply

    assert moved(both(lambda m: m["mask"].update(size=7))) > 0.05 and moved(both(lambda m: m["mask"].update(size=5))) > 0.05
    assert moved(both(lambda m: m.pop("mask"))) > 0.05 and moved(lambda c: attend(c)["mask"].update(size=7)) > 0.02
    assert moved(both(lambda m: m["rot"].update(dims=6))) > 0.05 and moved(both(lambda m: m["rot"].update(base=90.0))) > 0.02
    assert moved(both(lambda m: m.update(scale=0.6))) > 0.05
    assert moved(softmax_with_silent_key=lambda s: torch.softmax(s, 0)) > 0.05
    assert moved(rotate_halves=lambda x, dims, base: x) > 0.05
    assert moved(unit_vector=lambda x: x / 2.0) > 0.05
    assert moved(general_delta_decay=lambda h, t, p: torch.full((h.shape[0], t[p + "w0"].shape[0]), 0.8, dtype=h.dtype)) > 0.05
    assert moved(poly_norm=lambda z, c, eps: c[0] * z + c[1] * z ** 2 + c[2] * z ** 3 + c[3]) > 0.05
    # (a factor on a token's whole mixture would not show: the norm behind it takes it out again)
    assert moved(choose_experts=lambda z, top: (z.topk(top).indices, torch.full((z.shape[0], top), 1.0 / top, dtype=z.dtype))) > 0.05
    assert moved(choose_experts=lambda z, top: (lambda v, i: (i, torch.softmax(v, -1)))(*(-z).topk(top))) > 0.05
    for name in ("l0.mix.a.b", "l0.mix.w0", "l1.mix.z.b", "l1.mix.x.b", "l0.mlp.act", "l2.norm1b", "l2.norm2b", "l3.mix.norm"):
        assert moved(change_weights=lambda w: w.update({name: w[name].flip(0)})) > 0.02, name
    shifted = plain.forward(config, weights, tokens[1:])  # one token less: states, windows and positions all differ
    assert float((right[-1] - shifted[-1]).abs().max()) > 0.02


@pytest.mark.parametrize("name,cuts", [("E", (260,)), ("E", (3, 1, 252, 2, 1, 1)), ("E", (4, 4, 248) + (1,) * 4), ("A", (16, 15, 1, 96, 2) + (1,) * 10)])
def test_what_a_loud_first_token_wrote_is_read_far_later(tmp_path, name, cuts):
    """A state that is dropped, zeroed or not carried over a portion's or a page's border loses the first token: two prompts
    that differ in it only give different logits at their end, and the framework agrees with the plain model on both, however
    the prompt is cut (first portions that end inside the first page, at its border, behind it)."""
    config = CONFIGS[name]
    weights = long_memory(random_weights(config, 4))
    folder = write_folder(tmp_path / name, config, seed=4, weights=weights)
    config, tensors = plain.read_folder(folder)
    n = sum(cuts)
    base = prompts(config["vocab"], [n], seed=9)["r0"]
    other = [(base[0] + 1) % config["vocab"]] + base[1:]
    want = {rid: logits_of(config, tensors, toks)[-4:] for rid, toks in (("base", base), ("other", other))}
    assert float((want["base"] - want["other"]).abs().max()) > 0.02  # the far token shows
    page = PAGE_SIZE[name]
    for rid, toks in (("base", base), ("other", other)):
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
    """A short prompt and then 120 tokens one by one: the windows pass over decoded tokens only, pages behind them go back
    to the pool (which is smaller than the sequence), the states are carried 120 times."""
    folder = write_folder(tmp_path / "A", CONFIGS["A"], seed=6)
    config, weights = plain.read_folder(folder)
    toks = prompts(config["vocab"], [123], seed=12)["r0"]
    want = logits_of(config, weights, toks)
    replayer = Replayer(folder, "float32", 124, block_size=4, device="cpu", ops=TorchOps(), max_live=1)
    rows = [torch.from_numpy(replayer.step({"step": 0, "entries": [{"id": "a", "tokens": toks[:3], "want": [0, 1, 2]}], "end": []}))]
    for i in range(3, 123):
        rows.append(torch.from_numpy(replayer.step({"step": i, "entries": [{"id": "a", "tokens": [toks[i]], "want": [0]}], "end": ["a"] if i == 122 else []})))
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
    if name == "A":
        tight = engine_for(num_gpu_blocks=11)
        assert [r.output_token_ids for r in tight.generate(requests("t"))] == want
        assert tight.cache.num_used_pages() == 0
        tight.cache.assert_consistent([])
