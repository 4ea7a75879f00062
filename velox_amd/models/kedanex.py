"""Kedanex as a ``ModelSpec``.

A decoder with a norm before and one behind every sub-layer (``x += norm1b(mixer(norm1(x))); x += norm2b(ff(norm2(x)))``, RMS
norms with weights; ``parts.block.SandwichBlock``).  ``config.json`` lists the layers one by one, each with its type and sizes,
so layers may differ in everything; a layer that says ``weights_of: j`` is layer ``j``'s block run again with a cache or state
of its own.  Three types of mixer, each with any of the feed-forwards:

``general_delta``
    the generalized delta rule: a matrix per head with a decay and a removal rate per key channel, which removes what
    it holds along the key's direction and writes the key itself (``parts.linear_recurrence.GeneralDeltaMixer``).
``mingru``
    a gated recurrence on every channel by itself with gates that do not depend on the state (``parts.gated_recurrence``).
``attention``
    grouped-query softmax attention over a sliding window whose values are the keys as projected, with a rotation of the
    first ``rot.dims`` channels, queries and keys divided by their root mean square behind the rotation, the score scale of
    the configuration and a silent key of score 0 in every softmax (``parts.conv_attention``).

The feed-forward is ``W_down polynorm(W_up h)`` (``dense``), a mixture of gated SiLU experts whose weights are the softmax over the
chosen logits (``moe``), or absent.

Tensor names: ``embed``, ``head``, ``final.norm``, and per layer ``l<i>.norm{1,1b,2,2b}``, ``l<i>.mix.*`` as the mixers' parts name them,
``l<i>.mlp.{up,down,act}`` or ``l<i>.mlp.{router,e<k>.gate,e<k>.up,e<k>.down}``.  The inner size of the decay's low-rank map is a
size that only the tensors' shapes give.  There is no position limit in the configuration, so ``max_position`` is the caller's.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from ..config.model_config import ConfigError, ModelConfig, require
from ..config.registry import architecture_name, register_architecture
from ..parts import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

# positions an engine is given when its caller names no limit (the configuration has none)
DEFAULT_MAX_POSITION = 1 << 17
SINK_SCORE = 0.0  # the score of the key without a value in every softmax
_TYPES = ("general_delta", "mingru", "attention")


def _section(raw: Dict[str, Any], key: str, where: str) -> Dict[str, Any]:
    value = raw.get(key)
    if not isinstance(value, dict):
        raise ConfigError(f"config.json: {where}{key!r} must be an object")
    return value


def _attention(mixer: Dict[str, Any], where: str) -> Dict[str, Any]:
    out: Dict[str, Any] = {key: require(mixer, key, int) for key in ("heads", "kv_heads", "dim", "vdim")}
    if min(out.values()) <= 0 or out["heads"] % out["kv_heads"]:
        raise ConfigError(f"{where}: heads, kv_heads, dim and vdim must be positive and heads a multiple of kv_heads")
    if out["vdim"] != out["dim"]:
        raise ConfigError(f"{where}: values are the keys, so vdim={out['vdim']} must equal dim={out['dim']}")
    out["scale"] = require(mixer, "scale", float)
    if not out["scale"] > 0:
        raise ConfigError(f"{where}.scale must be positive")
    out["window"] = None
    if mixer.get("mask") is not None:
        out["window"] = require(_section(mixer, "mask", where + "."), "size", int)
        if out["window"] < 1:
            raise ConfigError(f"{where}.mask.size must be at least 1")
    out["rotation"] = None
    if mixer.get("rot") is not None:
        rot = _section(mixer, "rot", where + ".")
        dims, base = require(rot, "dims", int), require(rot, "base", float)
        if dims < 0 or dims % 2 or dims > out["dim"] or not base > 0:
            raise ConfigError(f"{where}.rot: dims={dims} must be even and at most dim={out['dim']}, base positive")
        if dims:
            out["rotation"] = (dims, base)
    return out


def _general_delta(mixer: Dict[str, Any], where: str, shapes: Dict[str, Any], low_rank_name: str) -> Dict[str, Any]:
    out = {key: require(mixer, key, int) for key in ("heads", "dim")}
    # the rows of the decay map's first half: a folder's reader notes the shapes, a configuration without a folder states ``w1_rank``
    if low_rank_name in shapes:
        out["rank"] = int(shapes[low_rank_name][0])
    elif mixer.get("w1_rank") is not None:
        out["rank"] = int(mixer["w1_rank"])
    else:
        raise ConfigError(f"{where}: the inner size of the decay's low-rank map is the first size of tensor {low_rank_name!r}; "
                          "read the configuration from a model folder or state 'w1_rank'")
    if min(out.values()) <= 0:
        raise ConfigError(f"{where}: heads, dim and the inner size of the decay's low-rank map must be positive")
    return out


def _mingru(mixer: Dict[str, Any], where: str) -> Dict[str, Any]:
    out = {"width": require(mixer, "width", int)}
    if out["width"] <= 0:
        raise ConfigError(f"{where}.width must be positive")
    return out


def _feed_forward(mlp: Optional[Dict[str, Any]], where: str) -> Optional[Dict[str, Any]]:
    if mlp is None:
        return None
    kind = mlp.get("kind")
    if kind == "dense":
        out = {"kind": "dense", "ff": require(mlp, "ff", int)}
    elif kind == "moe":
        router = _section(mlp, "router", where + "mlp.")
        out = {"kind": "moe", "ff": require(_section(mlp, "expert", where + "mlp."), "ff", int), "experts": require(router, "experts", int),
               "top": require(router, "top", int)}
        if not 1 <= out["top"] <= out["experts"]:
            raise ConfigError(f"{where}mlp.router: top={out['top']} must lie between 1 and experts={out['experts']}")
    else:
        raise ConfigError(f"{where}mlp.kind={kind!r} is not a feed-forward of this design ('dense' or 'moe')")
    if out["ff"] <= 0:
        raise ConfigError(f"{where}mlp: ff must be positive")
    return out


@dataclass
class KedanexConfig(ModelConfig):
    width: int = 0
    vocab: int = 0
    norm_eps: float = 0.0
    layers: List[Dict[str, Any]] = field(default_factory=list)  # validated copies of the entries; "owner" = whose tensors a layer runs

    @staticmethod
    def from_dict(raw: Dict[str, Any]) -> "KedanexConfig":
        width, vocab = require(raw, "width", int), require(raw, "vocab", int)
        eps = require(_section(raw, "norm", ""), "eps", float)
        if width <= 0 or vocab <= 0 or not eps > 0:
            raise ConfigError("width, vocab and norm.eps must be positive")
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError("config.json: 'layers' must list at least one layer")
        shapes = raw.get("tensor_shapes") or {}
        owners: List[int] = []  # whose tensors a layer runs: itself, or the layer its ``weights_of`` leads to
        for index, entry in enumerate(listed):
            if not isinstance(entry, dict) or entry.get("type") not in _TYPES:
                raise ConfigError(f"layers[{index}].type={entry.get('type') if isinstance(entry, dict) else entry!r} is not a layer of this design ({', '.join(_TYPES)})")
            owner, seen = index, set()
            while listed[owner].get("weights_of") is not None:
                seen.add(owner)
                owner = int(listed[owner]["weights_of"])
                if not 0 <= owner < len(listed) or owner in seen or not isinstance(listed[owner], dict):
                    raise ConfigError(f"layers[{index}].weights_of must lead to a layer that owns its tensors")
            if listed[owner].get("type") != entry["type"]:
                raise ConfigError(f"layers[{index}]: a layer that runs layer {owner}'s weights is of its type")
            owners.append(owner)
        layers: List[Dict[str, Any]] = [{} for _ in listed]
        for index, entry in enumerate(listed):
            if owners[index] != index:
                continue
            where, kind = f"layers[{index}].", entry["type"]
            mixer = _section(entry, "mixer", where)
            if kind == "attention":
                parsed = _attention(mixer, where + "mixer")
            elif kind == "general_delta":
                parsed = _general_delta(mixer, where + "mixer", shapes, f"l{index}.mix.w1")
            else:
                parsed = _mingru(mixer, where + "mixer")
            layers[index] = {"type": kind, "owner": index, "mixer": parsed, "mlp": _feed_forward(entry.get("mlp"), where)}
        for index, owner in enumerate(owners):
            if owner != index:
                layers[index] = dict(layers[owner], owner=owner)
        return KedanexConfig(architecture=architecture_name(raw), raw=dict(raw), width=width, vocab=vocab, norm_eps=eps, layers=layers)

    def to_json_dict(self) -> Dict[str, Any]:
        return {key: value for key, value in self.raw.items() if key != "tensor_shapes"}


def kedanex_spec(config: KedanexConfig, max_position: Optional[int] = None) -> ModelSpec:
    max_position = int(max_position or DEFAULT_MAX_POSITION)
    width, eps = config.width, config.norm_eps
    norm = PartSpec.of("rmsnorm", hidden_size=width, eps=eps, weight_name="")
    positions: Dict[str, PartSpec] = {}
    layers: List[LayerSpec] = []
    place: Dict[int, int] = {}  # configuration index of a weight-owning layer -> its place in ``layers``
    for index, layer in enumerate(config.layers):
        if layer["owner"] != index:
            continue
        sizes, position = layer["mixer"], None
        if layer["type"] == "attention":
            if sizes["rotation"] is not None:
                dims, base = sizes["rotation"]
                position = f"rot_{dims}_{base!r}"  # (layers with the same rotation share its tables)
                positions.setdefault(position, PartSpec.of("rotary", rotary_dim=dims, theta=base, max_position=max_position, exact_angles=True))
            mixer = PartSpec.of("conv_attention", hidden_size=width, num_heads=sizes["heads"], num_kv_heads=sizes["kv_heads"], dim=sizes["dim"],
                                vdim=sizes["vdim"], scale=sizes["scale"], window=sizes["window"], conv_taps=0, qkv_bias=False, out_bias=False,
                                post_norm_eps=eps, values_are_keys=True, sink_score=SINK_SCORE)
        elif layer["type"] == "general_delta":
            mixer = PartSpec.of("general_delta", hidden_size=width, num_heads=sizes["heads"], dim=sizes["dim"], vdim=sizes["dim"], norm_eps=eps,
                                decay_rank=sizes["rank"])
        else:
            mixer = PartSpec.of("gated_recurrence", hidden_size=width, width=sizes["width"], shift=0.5)
        mlp = layer["mlp"]
        if mlp is None:
            feed_forward = PartSpec.of("none")
        elif mlp["kind"] == "dense":
            feed_forward = PartSpec.of("plain_mlp", hidden_size=width, intermediate_size=mlp["ff"], activation="poly_norm", names=("up", "down"), norm_eps=eps,
                                       coefficients_name="act")
        else:
            # (the softmax over the chosen logits is the softmax over all of them, divided by the sum of the chosen)
            feed_forward = PartSpec.of("routed_experts", hidden_size=width, intermediate_size=mlp["ff"], num_experts=mlp["experts"], top=mlp["top"],
                                       score="softmax", renormalize=True, scale_input=False, expert_names=("e{e}.gate", "e{e}.up", "e{e}.down"),
                                       router_name="router")
        place[index] = len(layers)
        layers.append(LayerSpec(prefix=f"l{index}.", mixer=mixer, feed_forward=feed_forward, mixer_norm=norm, ff_norm=norm, position=position,
                                arrangement="sandwich", arrangement_args=(("output_norm", norm), ("output_norm_prefixes", ("norm1b", "norm2b"))),
                                mixer_prefix="mix.", feed_forward_prefix="mlp.", mixer_norm_prefix="norm1", ff_norm_prefix="norm2"))
    schedule = [ScheduleEntry(place[layer["owner"]]) for layer in config.layers]
    return ModelSpec(vocab_size=config.vocab, hidden_size=width, max_position=max_position, layers=layers, schedule=schedule, final_norm=norm,
                     positions=positions, tie_head=False, embed_name="embed", head_name="head", final_norm_prefix="final.norm", eos_token_ids=())


register_architecture("Kedanex", KedanexConfig.from_dict, kedanex_spec, reads_tensor_shapes=True)
