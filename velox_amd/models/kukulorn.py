"""Kukulorn as a ``ModelSpec``.

A decoder whose layers have one norm and two sub-layers side by side, ``x += mixer(norm(x)) + ff(norm(x))`` (RMS norms with weights;
``parts.block.ParallelBlock``).  ``config.json`` lists the layers one by one, each with its type and sizes, so layers may differ in
everything.  With a ``loop`` the layers ``start .. stop - 1`` run ``times`` times in a row with the same weights, every pass with caches
and states of its own; before the first layer of every pass the residual becomes ``W [x; x0]`` with ``x0`` the embedding output
(``parts.model.LinearPassInput``).  Two types of layer:

``attention``
    grouped-query softmax attention over all keys with biases on q, k and v, a short causal convolution on them, a rotation of the
    first ``rot.dims`` channels whose slow frequencies are stretched by wavelength, queries and keys divided by their root mean
    square behind the rotation, capped scores and a gate per channel on the heads' outputs (``parts.conv_attention``);
``parallel``
    two mixers on the same input (``parts.parallel_mixer``), each output normed over the width with a weight of its own, half their
    sum: on the left grouped-query attention with biases, queries and keys normed over the whole projection, a learned bias by
    distance, a sliding window that keeps the sequence's first tokens, and a gate per head (``parts.normed_attention``); on the
    right a selective state space (``parts.state_space``).

The feed-forward is ``W_down (relu(W_gate h) * W_up h)`` or absent.  Logits are the product with the embedding table, capped.

Tensor names: ``embed``, ``loop.in``, ``final.norm``, and per layer ``l<i>.norm1``, ``l<i>.mix.*`` as the mixers' parts name them (below
``left.`` / ``right.`` in a parallel layer, whose norms are ``left.out`` / ``right.out``), ``l<i>.mlp.{gate,up,down}``.  The number of distance
buckets is a size that only the tensors' shapes give.  There is no position limit in the configuration, so ``max_position`` is the
caller's.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from ..config.model_config import ConfigError, ModelConfig, require
from ..config.registry import architecture_name, register_architecture
from ..parts import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

# positions an engine is given when its caller names no limit (the configuration has none)
DEFAULT_MAX_POSITION = 1 << 17
OUTPUT_SHARE = 0.5  # of each of a parallel layer's two normed outputs
_TYPES = ("attention", "parallel")


def _section(raw: Dict[str, Any], key: str, where: str) -> Dict[str, Any]:
    value = raw.get(key)
    if not isinstance(value, dict):
        raise ConfigError(f"config.json: {where}{key!r} must be an object")
    return value


def _heads(mixer: Dict[str, Any], where: str) -> Dict[str, Any]:
    out: Dict[str, Any] = {key: require(mixer, key, int) for key in ("heads", "kv_heads", "dim", "vdim")}
    if min(out.values()) <= 0 or out["heads"] % out["kv_heads"]:
        raise ConfigError(f"{where}: heads, kv_heads, dim and vdim must be positive and heads a multiple of kv_heads")
    out["scale"] = require(mixer, "scale", float)
    if not out["scale"] > 0:
        raise ConfigError(f"{where}.scale must be positive")
    return out


def _rotation(mixer: Dict[str, Any], where: str, limit: int) -> Optional[tuple]:
    """``(dims, base, (factor, low, high, original) or None)`` of a mixer's ``rot`` entry, or None when nothing is rotated."""
    if mixer.get("rot") is None:
        return None
    rot = _section(mixer, "rot", where + ".")
    dims, base = require(rot, "dims", int), require(rot, "base", float)
    if dims < 0 or dims % 2 or dims > limit or not base > 0:
        raise ConfigError(f"{where}.rot: dims={dims} must be even and at most dim={limit}, base positive")
    bands = None
    if rot.get("scaling") is not None:
        scaling = _section(rot, "scaling", where + ".rot.")
        bands = tuple(require(scaling, key, float) for key in ("factor", "low", "high", "original"))
        if not min(bands) > 0 or not bands[2] > bands[1]:
            raise ConfigError(f"{where}.rot.scaling: factor, low, high and original must be positive and high above low")
    return (dims, base, bands) if dims else None


def _attention(mixer: Dict[str, Any], where: str) -> Dict[str, Any]:
    out = _heads(mixer, where)
    out["conv"] = int(mixer.get("conv") or 0)
    out["softcap"] = float(mixer["softcap"]) if mixer.get("softcap") is not None else None
    if out["conv"] < 0 or (out["softcap"] is not None and not out["softcap"] > 0):
        raise ConfigError(f"{where}: conv must not be negative, softcap must be positive")
    out["rotation"] = _rotation(mixer, where, out["dim"])
    return out


def _kept_window(mixer: Dict[str, Any], where: str, shapes: Dict[str, Any], table: str) -> Dict[str, Any]:
    out = _heads(mixer, where)
    out["window"], out["keep_first"] = None, 0
    if mixer.get("mask") is not None:
        mask = _section(mixer, "mask", where + ".")
        out["window"], out["keep_first"] = require(mask, "size", int), int(mask.get("keep_first") or 0)
        if out["window"] < 1 or out["keep_first"] < 0:
            raise ConfigError(f"{where}.mask: size must be at least 1, keep_first not negative")
    # rows of the bias table: a folder's reader notes the shapes, a configuration without a folder states ``buckets``
    if table in shapes:
        out["buckets"] = int(shapes[table][0])
    elif mixer.get("buckets") is not None:
        out["buckets"] = int(mixer["buckets"])
    else:
        raise ConfigError(f"{where}: the number of distance buckets is the first size of tensor {table!r}; read the configuration from a model "
                          "folder or state 'buckets'")
    out["far"] = require(mixer, "bias_max", float)
    if out["buckets"] < 1 or not out["far"] > 0:
        raise ConfigError(f"{where}: the bias needs at least one bucket and a positive bias_max")
    return out


def _state_space(mixer: Dict[str, Any], where: str) -> Dict[str, Any]:
    out = {key: require(mixer, key, int) for key in ("heads", "groups", "state", "vdim", "conv", "norm_groups")}
    if min(out.values()) <= 0 or out["heads"] % out["groups"] or out["heads"] * out["vdim"] % out["norm_groups"]:
        raise ConfigError(f"{where}: heads, groups, state, vdim, conv and norm_groups must be positive, heads a multiple of groups and "
                          "heads * vdim a multiple of norm_groups")
    return out


def _loop(raw: Dict[str, Any], count: int) -> Optional[tuple]:
    """``(start, stop, times)``, or None when every layer runs once and nothing stands before a pass."""
    if raw.get("loop") is None:
        return None
    loop = _section(raw, "loop", "")
    start, stop, times = (require(loop, key, int) for key in ("start", "stop", "times"))
    if not 0 <= start < stop <= count or times < 1:
        raise ConfigError(f"config.json: loop must run at least one of the {count} layers at least once (start={start}, stop={stop}, times={times})")
    return start, stop, times


@dataclass
class KukulornConfig(ModelConfig):
    width: int = 0
    vocab: int = 0
    norm_eps: float = 0.0
    logit_softcap: Optional[float] = None
    loop: Optional[tuple] = None  # (start, stop, times)
    layers: List[Dict[str, Any]] = field(default_factory=list)  # validated copies of the configuration's entries

    @staticmethod
    def from_dict(raw: Dict[str, Any]) -> "KukulornConfig":
        width, vocab = require(raw, "width", int), require(raw, "vocab", int)
        eps = require(_section(raw, "norm", ""), "eps", float)
        if width <= 0 or vocab <= 0 or not eps > 0:
            raise ConfigError("width, vocab and norm.eps must be positive")
        softcap = float(raw["logit_softcap"]) if raw.get("logit_softcap") is not None else None
        if softcap is not None and not softcap > 0:
            raise ConfigError("logit_softcap must be positive")
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError("config.json: 'layers' must list at least one layer")
        shapes = raw.get("tensor_shapes") or {}
        layers: List[Dict[str, Any]] = []
        for index, entry in enumerate(listed):
            where = f"layers[{index}]"
            if not isinstance(entry, dict) or entry.get("type") not in _TYPES:
                raise ConfigError(f"{where}.type={entry.get('type') if isinstance(entry, dict) else entry!r} is not a layer of this design ({', '.join(_TYPES)})")
            mixer = _section(entry, "mixer", where + ".")
            parsed: Dict[str, Any] = {"type": entry["type"], "ff": None}
            if entry["type"] == "attention":
                parsed["mixer"] = _attention(mixer, where + ".mixer")
            else:
                parsed["left"] = _kept_window(_section(mixer, "left", where + ".mixer."), where + ".mixer.left", shapes, f"l{index}.mix.left.rel")
                parsed["right"] = _state_space(_section(mixer, "right", where + ".mixer."), where + ".mixer.right")
            mlp = entry.get("mlp")
            if mlp is not None:
                if mlp.get("kind") != "dense":
                    raise ConfigError(f"{where}.mlp.kind={mlp.get('kind')!r} is not a feed-forward of this design (only 'dense')")
                parsed["ff"] = require(mlp, "ff", int)
                if parsed["ff"] <= 0:
                    raise ConfigError(f"{where}.mlp.ff must be positive")
            layers.append(parsed)
        return KukulornConfig(architecture=architecture_name(raw), raw=dict(raw), width=width, vocab=vocab, norm_eps=eps, logit_softcap=softcap,
                              loop=_loop(raw, len(layers)), layers=layers)

    def to_json_dict(self) -> Dict[str, Any]:
        return {key: value for key, value in self.raw.items() if key != "tensor_shapes"}


def run_order(count: int, loop: Optional[tuple]) -> List[ScheduleEntry]:
    """The layers in the order of their runs."""
    if loop is None:
        return [ScheduleEntry(index) for index in range(count)]
    start, stop, times = loop
    passes = [ScheduleEntry(index, begins_pass=index == start) for _ in range(times) for index in range(start, stop)]
    return [ScheduleEntry(index) for index in range(start)] + passes + [ScheduleEntry(index) for index in range(stop, count)]


def kukulorn_spec(config: KukulornConfig, max_position: Optional[int] = None) -> ModelSpec:
    max_position = int(max_position or DEFAULT_MAX_POSITION)
    width, eps = config.width, config.norm_eps
    norm = PartSpec.of("rmsnorm", hidden_size=width, eps=eps, weight_name="")
    positions: Dict[str, PartSpec] = {}
    layers: List[LayerSpec] = []
    for index, layer in enumerate(config.layers):
        position = None
        if layer["type"] == "attention":
            sizes = layer["mixer"]
            if sizes["rotation"] is not None:
                dims, base, bands = sizes["rotation"]
                position = f"rot_{dims}_{base!r}_{bands!r}"  # (layers with the same rotation share its tables)
                positions.setdefault(position, PartSpec.of("rotary", rotary_dim=dims, theta=base, max_position=max_position, exact_angles=True, bands=bands))
            mixer = PartSpec.of("conv_attention", hidden_size=width, num_heads=sizes["heads"], num_kv_heads=sizes["kv_heads"], dim=sizes["dim"],
                                vdim=sizes["vdim"], scale=sizes["scale"], conv_taps=sizes["conv"], qkv_bias=True, out_bias=False, post_norm_eps=eps,
                                softcap=sizes["softcap"], gate="channel")
        else:
            sizes, right = layer["left"], layer["right"]
            left = PartSpec.of("normed_attention", hidden_size=width, num_heads=sizes["heads"], num_kv_heads=sizes["kv_heads"], dim=sizes["dim"],
                               vdim=sizes["vdim"], scale=sizes["scale"], norm_eps=eps, qk_norm="whole", distance_bias=(sizes["buckets"], sizes["far"]),
                               qkv_bias=True, out_bias=True, window=sizes["window"], keep_first=sizes["keep_first"], gate="head",
                               names=(("q", "q"), ("k", "k"), ("v", "v"), ("o", "o"), ("q_norm", "q.norm"), ("k_norm", "k.norm"), ("rel", "rel"), ("gate", "g")))
            state_space = PartSpec.of("state_space", hidden_size=width, num_heads=right["heads"], groups=right["groups"], state=right["state"],
                                      vdim=right["vdim"], conv_taps=right["conv"], norm_groups=right["norm_groups"], norm_eps=eps)
            mixer = PartSpec.of("parallel_mixers", left=left, right=state_space, left_scale=OUTPUT_SHARE, right_scale=OUTPUT_SHARE, output_norm=norm)
        if layer["ff"] is None:
            feed_forward = PartSpec.of("none")
        else:
            feed_forward = PartSpec.of("gated_mlp", hidden_size=width, intermediate_size=layer["ff"], activation="relu", names=("gate", "up", "down"))
        layers.append(LayerSpec(prefix=f"l{index}.", mixer=mixer, feed_forward=feed_forward, mixer_norm=norm, ff_norm=norm, position=position,
                                arrangement="parallel", mixer_prefix="mix.", feed_forward_prefix="mlp.", mixer_norm_prefix="norm1", ff_norm_prefix="norm1"))
    return ModelSpec(vocab_size=config.vocab, hidden_size=width, max_position=max_position, layers=layers, schedule=run_order(len(layers), config.loop),
                     final_norm=norm, positions=positions, tie_head=True, embed_name="embed", head_name="head", final_norm_prefix="final.norm",
                     eos_token_ids=(), head=PartSpec.of("linear", softcap=config.logit_softcap),
                     pass_input=PartSpec.of("linear", name="loop.in") if config.loop is not None else None)


register_architecture("Kukulorn", KukulornConfig.from_dict, kukulorn_spec, reads_tensor_shapes=True)
