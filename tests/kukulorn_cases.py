"""Small Kukulorn configurations and weights for the tests, written here from the design's tensor names and shapes (not
from the framework's tables, so that a wrong name or shape there shows).  The weights are sharp: attention is peaked by its
scale, the bias by distance and the norms' weights are spread, decays lie between "forgets within two tokens" and "keeps for
hundreds", gates are spread.  A key that is lost, a window that is one off, a kept token that is not seen, a state that is not
carried or a norm left out then changes the logits by far more than any tolerance."""
from __future__ import annotations

import json
import os
from typing import Dict, List, Optional

import torch
from safetensors.torch import save_file


def attention(heads: int, kv_heads: int, dim: int, vdim: int, scale: float, conv: int = 3, softcap: Optional[float] = 4.0, rot=None) -> dict:
    """``rot``: (dims, base) or (dims, base, factor, low, high, original)."""
    out = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "conv": conv}
    if softcap is not None:
        out["softcap"] = softcap
    if rot is not None:
        out["rot"] = {"dims": rot[0], "base": rot[1]}
        if len(rot) > 2:
            out["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), rot[2:]))
    return out


def left(heads: int, kv_heads: int, dim: int, vdim: int, scale: float, buckets: int, bias_max: float, window: Optional[int] = None, keep_first: int = 0) -> dict:
    """``buckets``: rows of the bias table, a size that only the tensors give (it stands here where no folder is at hand)."""
    out = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "buckets": buckets, "bias_max": bias_max}
    if window is not None:
        out["mask"] = {"size": window, "keep_first": keep_first}
    return out


def right(heads: int, groups: int, state: int, vdim: int, conv: int, norm_groups: int) -> dict:
    return {"heads": heads, "groups": groups, "state": state, "vdim": vdim, "conv": conv, "norm_groups": norm_groups}


def layer(mixer: dict, ff: Optional[int], other: Optional[dict] = None) -> dict:
    mlp = {"kind": "dense", "ff": ff} if ff is not None else None
    if other is None:
        return {"type": "attention", "mixer": mixer, "mlp": mlp}
    return {"type": "parallel", "mixer": {"left": mixer, "right": other}, "mlp": mlp}


def model(vocab: int, width: int, layers: List[dict], loop=None, eps: float = 1e-5, softcap: Optional[float] = 6.0) -> dict:
    out = {"architecture": "Kukulorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    if softcap is not None:
        out["logit_softcap"] = softcap
    return out


# Sizes that differ wherever two could be told apart: the loop starts and ends inside the list and crosses a layer of each type, value
# heads smaller and larger than key heads, windows and kept tokens that end inside, at and beyond pages of 4, a layer without a
# feed-forward inside the loop, both kinds of rotation.
CONFIG_A = model(97, 64, [
    layer(attention(4, 2, 16, 12, 0.8, conv=3, rot=(8, 100.0, 4.0, 1.0, 4.0, 40)), 40),
    layer(left(6, 2, 12, 20, 0.9, 10, 30.0, window=7, keep_first=3), 56, right(3, 1, 10, 12, 4, 2)),
    layer(attention(3, 3, 20, 24, 0.6, conv=2, softcap=2.5, rot=(20, 50.0)), None),
    layer(left(4, 4, 16, 16, 0.7, 7, 14.0, window=9, keep_first=5), 36, right(4, 2, 16, 10, 2, 4)),
    layer(left(2, 1, 24, 16, 0.8, 16, 100.0), 48, right(2, 2, 6, 20, 3, 1)),
], loop=(1, 3, 3))
# Nothing a multiple of 4, 8 or 16 where it need not be; no loop, no caps; more query heads to a key head than a tile has rows; a window
# that keeps nothing.
CONFIG_B = model(131, 86, [
    layer(left(6, 2, 10, 14, 0.9, 9, 22.0, window=11, keep_first=0), 22, right(3, 3, 9, 7, 5, 3)),
    layer(attention(5, 1, 14, 10, 0.9, conv=4, softcap=None, rot=(6, 30.0)), 22),
    layer(left(20, 1, 6, 6, 0.8, 5, 9.0, window=4, keep_first=2), None, right(2, 1, 33, 5, 2, 2)),
], eps=3e-6, softcap=None)
# Sizes the kernels for decode-sized bfloat16 batches and the matrix cores take (multiples of 64 and 16); a state of more entries than
# a workgroup of the chunked kernels holds at a time and columns of more than one slice; the whole list is the loop.
CONFIG_C = model(160, 128, [
    layer(left(8, 2, 64, 64, 0.25, 12, 60.0, window=24, keep_first=20), 192, right(4, 2, 64, 32, 4, 2)),
    layer(attention(8, 2, 64, 64, 0.3, conv=4, softcap=5.0, rot=(32, 10000.0, 8.0, 1.0, 4.0, 64)), 128),
    layer(left(4, 4, 128, 128, 0.2, 8, 40.0, window=40, keep_first=17), None, right(2, 1, 160, 80, 3, 1)),
], loop=(0, 3, 2))
# What other configurations make differ is equal or 1 here: one head everywhere, a window of one token beside one kept token, one
# bucket, one tap, one group, one pass of a loop of one layer.
CONFIG_D = model(64, 48, [
    layer(left(1, 1, 16, 16, 1.0, 1, 1.0, window=1, keep_first=1), 48, right(1, 1, 1, 48, 1, 1)),
    layer(attention(1, 1, 16, 16, 1.0, conv=1, rot=(16, 10.0)), 48),
], loop=(1, 2, 1), eps=1e-6)
# The kept tokens reach further than the window, and than the prompts' first portions.
CONFIG_E = model(80, 32, [
    layer(left(2, 2, 8, 8, 0.8, 6, 16.0, window=3, keep_first=13), 24, right(2, 1, 8, 8, 4, 2)),
    layer(attention(2, 1, 8, 8, 0.9, conv=3), 24),
], loop=(0, 1, 2))
CONFIGS = {"A": CONFIG_A, "B": CONFIG_B, "C": CONFIG_C, "D": CONFIG_D, "E": CONFIG_E}
PAGE_SIZE = {"A": 4, "B": 8, "C": 16, "D": 16, "E": 4}


def tensor_shapes(config: dict) -> Dict[str, tuple]:
    width = config["width"]
    shapes = {"embed": (config["vocab"], width), "final.norm": (width,)}
    if config.get("loop"):
        shapes["loop.in"] = (width, 2 * width)
    for i, entry in enumerate(config["layers"]):
        p = f"l{i}."
        shapes[p + "norm1"] = (width,)
        if entry["type"] == "attention":
            m, q = entry["mixer"], p + "mix."
        else:
            m, q = entry["mixer"]["left"], p + "mix.left."
        rows = {"q": m["heads"] * m["dim"], "k": m["kv_heads"] * m["dim"], "v": m["kv_heads"] * m["vdim"]}
        for name, n in rows.items():
            shapes[q + name], shapes[q + name + ".b"] = (n, width), (n,)
            if entry["type"] == "attention":
                shapes[q + name + ".conv"] = (n, m["conv"])
        shapes[q + "o"] = (width, m["heads"] * m["vdim"])
        if entry["type"] == "attention":
            shapes[q + "g"] = (m["heads"] * m["vdim"], width)
        else:
            shapes[q + "o.b"], shapes[q + "g"] = (width,), (m["heads"], width)
            shapes[q + "q.norm"], shapes[q + "k.norm"], shapes[q + "rel"] = (rows["q"],), (rows["k"],), (m["buckets"], m["heads"])
            m, q = entry["mixer"]["right"], p + "mix.right."
            inner, gn = m["heads"] * m["vdim"], m["groups"] * m["state"]
            shapes[q + "in"], shapes[q + "conv"], shapes[q + "conv.b"] = (2 * inner + 2 * gn + m["heads"], width), (inner + 2 * gn, m["conv"]), (inner + 2 * gn,)
            shapes[q + "dt_bias"] = shapes[q + "A_log"] = shapes[q + "D"] = (m["heads"],)
            shapes[q + "norm"], shapes[q + "o"] = (inner,), (width, inner)
            shapes[p + "mix.left.out"] = shapes[p + "mix.right.out"] = (width,)
        if entry["mlp"] is not None:
            ff = entry["mlp"]["ff"]
            shapes[p + "mlp.gate"], shapes[p + "mlp.up"], shapes[p + "mlp.down"] = (ff, width), (ff, width), (width, ff)
    return shapes


def random_weights(config: dict, seed: int) -> Dict[str, torch.Tensor]:
    """float32 tensors: matrices N(0, gain^2 / fan-in), biases and the table of the distances spread, step sizes and decay rates over
    two orders of magnitude, norm weights 1 + N(0, 0.1), the embedding N(0, 1)."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(config).items():
        last = name.rsplit(".", 1)[-1]
        if last == "dt_bias":
            out[name] = -2.0 + 2.0 * torch.randn(shape, generator=g)
        elif last == "A_log":
            out[name] = 1.2 * torch.randn(shape, generator=g)
        elif last == "D":
            out[name] = 0.5 + torch.rand(shape, generator=g)
        elif last == "rel":
            out[name] = 1.5 * torch.randn(shape, generator=g)
        elif last == "conv":
            out[name] = torch.randn(shape, generator=g) / shape[1] ** 0.5 + 0.3
        elif last == "b":
            out[name] = 0.4 * torch.randn(shape, generator=g)
        elif len(shape) == 1:
            out[name] = 1.0 + 0.1 * torch.randn(shape, generator=g)
        elif name == "embed":
            out[name] = torch.randn(shape, generator=g)
        else:
            gain = {"g": 1.5, "q": 1.5, "k": 1.5}.get(last, 1.0)
            out[name] = torch.randn(shape, generator=g) * (gain / shape[1] ** 0.5)
    return out


def long_memory(weights: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
    """Decays close to 1 over hundreds of tokens: what a loud early token wrote into a state is read far on."""
    out = dict(weights)
    for name, t in weights.items():
        if name.endswith("A_log"):
            out[name] = torch.full_like(t, -7.0)
        elif name.endswith("dt_bias"):
            out[name] = torch.full_like(t, -1.0)
    return out


def write_folder(path, config: dict, seed: int, dtype: str = "float32", weights: Optional[Dict[str, torch.Tensor]] = None) -> str:
    """The written configuration does not state the rows of the bias tables, as a folder from elsewhere would not: the reader
    has to take them from the tensors' shapes."""
    path = str(path)
    os.makedirs(path, exist_ok=True)
    weights = weights if weights is not None else random_weights(config, seed)
    storage = torch.float32 if dtype == "float32" else torch.bfloat16
    save_file({name: t.to(storage).contiguous() for name, t in weights.items()}, os.path.join(path, "model.safetensors"))
    written = json.loads(json.dumps(config))
    for entry in written["layers"]:
        if entry["type"] == "parallel":
            entry["mixer"]["left"].pop("buckets", None)
    with open(os.path.join(path, "config.json"), "w", encoding="utf-8") as handle:
        json.dump(written, handle)
    return path


def prompts(vocab: int, lengths, seed: int) -> Dict[str, List[int]]:
    g = torch.Generator().manual_seed(seed)
    return {f"r{i}": torch.randint(0, vocab, (n,), generator=g).tolist() for i, n in enumerate(lengths)}
