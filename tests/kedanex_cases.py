"""Small Kedanex configurations and weights for the tests, written here from the design's tensor names and shapes (not
from the framework's tables, so that a wrong name or shape there shows).  The weights are sharp: attention is peaked by
its scale, decays lie between "forgets within two tokens" and "keeps for hundreds", removal rates and gates are spread,
PolyNorm's four numbers differ, router logits are spread.  A key that is lost, a window that is one off, a state that is
not carried or a norm left out then changes the logits by far more than any tolerance."""
from __future__ import annotations

import json
import os
from typing import Dict, List, Optional

import torch
from safetensors.torch import save_file


def general_delta(heads: int, dim: int, rank: int) -> dict:
    """``rank``: the inner size of the decay's map, a size that only the tensors give (``w1_rank`` stands for it where no
    folder is at hand)."""
    return {"heads": heads, "dim": dim, "w1_rank": rank}


def mingru(width: int) -> dict:
    return {"width": width}


def attention(heads: int, kv_heads: int, dim: int, scale: float, window: Optional[int] = None, rot=None) -> dict:
    """``rot``: (dims, base)."""
    out = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if window is not None:
        out["mask"] = {"size": window}
    if rot is not None:
        out["rot"] = {"dims": rot[0], "base": rot[1]}
    return out


def dense(ff: int) -> dict:
    return {"kind": "dense", "ff": ff}


def moe(experts: int, top: int, ff: int) -> dict:
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def layer(kind: str, mixer: dict, mlp: Optional[dict], weights_of: Optional[int] = None) -> dict:
    out = {"type": kind, "mixer": mixer, "mlp": mlp}
    if weights_of is not None:
        out["weights_of"] = weights_of
    return out


# Sizes that differ wherever two could be told apart: heads that are no multiple of 16, a window of 6 (larger than a page of
# 4), part of every head rotated, a layer without a feed-forward, every mixer once run again with another layer's weights.
_A = [layer("general_delta", general_delta(3, 12, 5), dense(40)), layer("mingru", mingru(20), moe(6, 2, 16)),
      layer("attention", attention(4, 2, 16, 0.7, window=6, rot=(8, 100.0)), moe(5, 3, 24)), layer("general_delta", general_delta(2, 20, 7), None),
      layer("attention", attention(3, 3, 24, 0.5, window=9, rot=(24, 50.0)), dense(36))]
CONFIG_A = {"architecture": "Kedanex", "vocab": 97, "width": 64, "norm": {"eps": 1e-5},
            "layers": _A + [dict(_A[2], weights_of=2), dict(_A[1], weights_of=1), dict(_A[3], weights_of=3)]}
# Nothing a multiple of 4, 8 or 16 where it need not be; attention without a window and without a rotation; one expert of three.
CONFIG_B = {"architecture": "Kedanex", "vocab": 131, "width": 86, "norm": {"eps": 3e-6},
            "layers": [layer("attention", attention(6, 2, 10, 0.9), dense(22)), layer("mingru", mingru(33), moe(3, 1, 14)),
                       layer("general_delta", general_delta(3, 6, 3), moe(7, 7, 10)), layer("attention", attention(5, 1, 14, 0.6, window=11, rot=(6, 30.0)), None)]}
# Sizes the kernels for decode-sized bfloat16 batches and the matrix cores take (multiples of 64 and 8); key heads of 64 and 128
# channels; a query group of 20 heads on one key head.
_C = [layer("general_delta", general_delta(2, 64, 16), moe(8, 3, 64)), layer("attention", attention(4, 2, 64, 0.3, window=24, rot=(32, 10000.0)), dense(192)),
      layer("mingru", mingru(192), moe(4, 2, 32)), layer("general_delta", general_delta(1, 128, 24), dense(64)),
      layer("attention", attention(20, 1, 32, 0.4, window=40, rot=(32, 1000.0)), moe(4, 1, 64))]
CONFIG_C = {"architecture": "Kedanex", "vocab": 160, "width": 128, "norm": {"eps": 1e-5}, "layers": _C + [dict(_C[0], weights_of=0)]}
# What other configurations make differ is equal or 1 here: one head everywhere, a window of one token, one expert, an inner size of 1.
CONFIG_D = {"architecture": "Kedanex", "vocab": 64, "width": 48, "norm": {"eps": 1e-6},
            "layers": [layer("attention", attention(1, 1, 16, 1.0, window=1, rot=(16, 10.0)), moe(1, 1, 16)), layer("mingru", mingru(48), None),
                       layer("general_delta", general_delta(1, 48, 1), dense(48))]}
# No layer keeps pages: every mixer's memory is a state of fixed size.
CONFIG_E = {"architecture": "Kedanex", "vocab": 80, "width": 32, "norm": {"eps": 1e-5},
            "layers": [layer("general_delta", general_delta(2, 8, 4), dense(24)), layer("mingru", mingru(24), dense(24)),
                       layer("general_delta", general_delta(2, 8, 4), dense(24), weights_of=0)]}
CONFIGS = {"A": CONFIG_A, "B": CONFIG_B, "C": CONFIG_C, "D": CONFIG_D, "E": CONFIG_E}
PAGE_SIZE = {"A": 4, "B": 8, "C": 16, "D": 16, "E": 4}


def tensor_shapes(config: dict) -> Dict[str, tuple]:
    width = config["width"]
    shapes = {"embed": (config["vocab"], width), "head": (config["vocab"], width), "final.norm": (width,)}
    for i, entry in enumerate(config["layers"]):
        if entry.get("weights_of") is not None:
            continue
        m, p, q = entry["mixer"], f"l{i}.", f"l{i}.mix."
        shapes[p + "norm1"] = shapes[p + "norm1b"] = (width,)
        if entry["type"] == "general_delta":
            size = m["heads"] * m["dim"]
            for name in ("r", "k", "v", "a", "g"):
                shapes[q + name] = (size, width)
            shapes[q + "a.b"] = shapes[q + "w0"] = shapes[q + "norm"] = (size,)
            shapes[q + "w1"], shapes[q + "w2"], shapes[q + "o"] = (m["w1_rank"], width), (size, m["w1_rank"]), (width, size)
        elif entry["type"] == "mingru":
            for name in ("z", "x", "g"):
                shapes[q + name] = (m["width"], width)
            shapes[q + "z.b"] = shapes[q + "x.b"] = (m["width"],)
            shapes[q + "o"] = (width, m["width"])
        else:
            shapes[q + "q"], shapes[q + "k"] = (m["heads"] * m["dim"], width), (m["kv_heads"] * m["dim"], width)
            shapes[q + "o"] = (width, m["heads"] * m["dim"])
        mlp = entry["mlp"]
        if mlp is None:
            continue
        shapes[p + "norm2"] = shapes[p + "norm2b"] = (width,)
        if mlp["kind"] == "dense":
            shapes[p + "mlp.up"], shapes[p + "mlp.down"], shapes[p + "mlp.act"] = (mlp["ff"], width), (width, mlp["ff"]), (4,)
        else:
            ff = mlp["expert"]["ff"]
            shapes[p + "mlp.router"] = (mlp["router"]["experts"], width)
            for e in range(mlp["router"]["experts"]):
                shapes[f"{p}mlp.e{e}.gate"], shapes[f"{p}mlp.e{e}.up"], shapes[f"{p}mlp.e{e}.down"] = (ff, width), (ff, width), (width, ff)
    return shapes


def random_weights(config: dict, seed: int) -> Dict[str, torch.Tensor]:
    """float32 tensors: matrices N(0, gain^2 / fan-in) with larger gains where a decision is taken; biases of decays, removal
    rates and gates spread; norm weights 1 + N(0, 0.1); the embedding N(0, 1)."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(config).items():
        last = name.rsplit(".", 1)[-1]
        if last == "w0":
            out[name] = -2.0 + 2.0 * torch.randn(shape, generator=g)
        elif last == "act":
            out[name] = torch.tensor([0.8, -0.6, 0.5, 0.3]) + 0.2 * torch.randn(shape, generator=g)
        elif last == "b":
            out[name] = -1.0 + 1.2 * torch.randn(shape, generator=g)
        elif len(shape) == 1:
            out[name] = 1.0 + 0.1 * torch.randn(shape, generator=g)
        elif name == "embed":
            out[name] = torch.randn(shape, generator=g)
        else:
            gain = {"router": 2.5, "w1": 1.5, "w2": 1.5, "a": 1.5, "g": 1.5, "z": 1.5}.get(last, 1.0)
            out[name] = torch.randn(shape, generator=g) * (gain / shape[1] ** 0.5)
    return out


def long_memory(weights: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
    """Decays close to 1, removal rates and update gates close to 0: what a loud early token wrote is read hundreds of tokens on."""
    out = dict(weights)
    for name, t in weights.items():
        if name.endswith("mix.w0"):
            out[name] = torch.full_like(t, -9.0)
        elif name.endswith("mix.w2"):
            out[name] = 0.2 * t
        elif name.endswith("mix.a.b") or name.endswith("mix.z.b"):
            out[name] = torch.full_like(t, -7.0)
        elif name.endswith("mix.a") or name.endswith("mix.z"):
            out[name] = 0.3 * t
    return out


def write_folder(path, config: dict, seed: int, dtype: str = "float32", weights: Optional[Dict[str, torch.Tensor]] = None) -> str:
    """The written configuration does not state the inner sizes of the low-rank maps, as a folder from elsewhere would not:
    the reader has to take them from the tensors' shapes."""
    path = str(path)
    os.makedirs(path, exist_ok=True)
    weights = weights if weights is not None else random_weights(config, seed)
    storage = torch.float32 if dtype == "float32" else torch.bfloat16
    save_file({name: t.to(storage).contiguous() for name, t in weights.items()}, os.path.join(path, "model.safetensors"))
    written = json.loads(json.dumps(config))
    for entry in written["layers"]:
        entry["mixer"].pop("w1_rank", None)
    with open(os.path.join(path, "config.json"), "w", encoding="utf-8") as handle:
        json.dump(written, handle)
    return path


def prompts(vocab: int, lengths, seed: int) -> Dict[str, List[int]]:
    g = torch.Generator().manual_seed(seed)
    return {f"r{i}": torch.randint(0, vocab, (n,), generator=g).tolist() for i, n in enumerate(lengths)}
