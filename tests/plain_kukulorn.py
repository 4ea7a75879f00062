"""Kukulorn, written out plainly: whole sequences, no cache, token-by-token loops, one function per mechanism.

This is the yardstick of the tests.  It shares no code with ``velox_amd``: it takes the configuration as the dictionary
that ``config.json`` holds and the tensors by their checkpoint names, and runs in whatever float type the tensors have
(the tests hand it float64 copies).

Notation: ``n`` tokens; ``h`` is a sub-layer's input ``[n, width]``.
"""
from __future__ import annotations

import json
import math
import os
from typing import Dict, List, Optional

import torch

Tensors = Dict[str, torch.Tensor]


# ----------------------------------------------------------------------------------------------------------------------
# small pieces
# ----------------------------------------------------------------------------------------------------------------------
def over_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    return over_rms(x, eps) * weight


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def soft_cap(x: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(x / cap)


def causal_conv(u: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    """``u`` [n, channels], ``weight`` [channels, taps]; the last column meets the current token, zeros before the start."""
    n, taps = u.shape[0], weight.shape[1]
    out = torch.zeros_like(u)
    for t in range(n):
        for j in range(taps):
            source = t - (taps - 1) + j
            if source >= 0:
                out[t] += weight[:, j] * u[source]
    return out


def banded_frequencies(dims: int, base: float, scaling: Optional[dict]) -> List[float]:
    """``base^(-2i/dims)``; with ``scaling`` wavelengths above ``original / low`` are made ``factor`` times longer, those
    below ``original / high`` stay, and between the two a straight line in ``original / wavelength`` leads from one to the other."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling is not None:
            turns = scaling["original"] / (2.0 * math.pi / f)  # whole turns within the original length
            if turns < scaling["low"]:
                f = f / scaling["factor"]
            elif turns <= scaling["high"]:
                s = (turns - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return out


def rotate_halves(x: torch.Tensor, dims: int, base: float, scaling: Optional[dict]) -> torch.Tensor:
    """``x`` [n, heads, d]: channel ``i`` of the first ``dims`` is turned with channel ``i + dims / 2``; the rest passes."""
    half = dims // 2
    freq = torch.tensor(banded_frequencies(dims, base, scaling), dtype=torch.float64)
    angle = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * freq[None, :]
    cos, sin = angle.cos().to(x.dtype)[:, None, :], angle.sin().to(x.dtype)[:, None, :]
    first, second = x[..., :half], x[..., half:dims]
    return torch.cat([first * cos - second * sin, second * cos + first * sin, x[..., dims:]], dim=-1)


def distance_bucket(n: int, buckets: int, far: float) -> int:
    near = buckets // 2
    if n < near:
        return n
    if near < 1 or far <= near:
        return buckets - 1
    return min(buckets - 1, near + math.floor(math.log(n / near) / math.log(far / near) * (buckets - near)))


def visible(i: int, window: Optional[int], keep_first: int) -> List[int]:
    """The positions that position ``i`` sees: the last ``window`` up to itself (None: all) and the first ``keep_first``."""
    return [j for j in range(i + 1) if window is None or i - j < window or j < keep_first]


# ----------------------------------------------------------------------------------------------------------------------
# mixers
# ----------------------------------------------------------------------------------------------------------------------
def capped_attention_mixer(h: torch.Tensor, t: Tensors, p: str, c: dict, eps: float) -> torch.Tensor:
    n, heads, groups, dim, vdim = h.shape[0], c["heads"], c["kv_heads"], c["dim"], c["vdim"]

    def projected(name):
        u = h @ t[p + name].T + t[p + name + ".b"]
        return causal_conv(u, t[p + name + ".conv"]) if c.get("conv") else u

    q, k, v = projected("q").reshape(n, heads, dim), projected("k").reshape(n, groups, dim), projected("v").reshape(n, groups, vdim)
    if c.get("rot"):
        args = (c["rot"]["dims"], c["rot"]["base"], c["rot"].get("scaling"))
        q, k = rotate_halves(q, *args), rotate_halves(k, *args)
    q, k = over_rms(q, eps), over_rms(k, eps)
    out = torch.zeros(n, heads, vdim, dtype=h.dtype)
    for i in range(n):
        for a in range(heads):
            g = a // (heads // groups)
            scores = (k[:i + 1, g] @ q[i, a]) * c["scale"]
            if c.get("softcap"):
                scores = soft_cap(scores, c["softcap"])
            out[i, a] = torch.softmax(scores, dim=-1) @ v[:i + 1, g]
    gate = torch.sigmoid(h @ t[p + "g"].T)
    return (out.reshape(n, heads * vdim) * gate) @ t[p + "o"].T


def kept_window_attention(h: torch.Tensor, t: Tensors, p: str, c: dict, eps: float) -> torch.Tensor:
    n, heads, groups, dim, vdim = h.shape[0], c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q, k, v = (h @ t[p + name].T + t[p + name + ".b"] for name in ("q", "k", "v"))
    q = rms_norm(q, t[p + "q.norm"], eps).reshape(n, heads, dim)
    k = rms_norm(k, t[p + "k.norm"], eps).reshape(n, groups, dim)
    v = v.reshape(n, groups, vdim)
    rel = t[p + "rel"]
    mask = c.get("mask") or {}
    out = torch.zeros(n, heads, vdim, dtype=h.dtype)
    for i in range(n):
        seen = visible(i, mask.get("size"), mask.get("keep_first", 0))
        buckets = [distance_bucket(i - j, rel.shape[0], c["bias_max"]) for j in seen]
        for a in range(heads):
            g = a // (heads // groups)
            scores = (k[seen, g] @ q[i, a]) * c["scale"] + rel[buckets, a]
            out[i, a] = torch.softmax(scores, dim=-1) @ v[seen, g]
    out = out * torch.sigmoid(h @ t[p + "g"].T)[:, :, None]
    return out.reshape(n, heads * vdim) @ t[p + "o"].T + t[p + "o.b"]


def state_space_scan(x, b, c, step, rate, skip) -> torch.Tensor:
    """``x`` [n, heads, vdim], ``b``, ``c`` [n, groups, N], ``step`` [n, heads]; per head ``S <- exp(-rate step) S + step b x^T``,
    ``y = S^T c + skip x``."""
    n, heads, vdim = x.shape
    groups = b.shape[1]
    out = torch.zeros_like(x)
    for a in range(heads):
        g = a // (heads // groups)
        state = torch.zeros(b.shape[2], vdim, dtype=x.dtype)
        for i in range(n):
            state = torch.exp(-rate[a] * step[i, a]) * state + step[i, a] * torch.outer(b[i, g], x[i, a])
            out[i, a] = state.T @ c[i, g] + skip[a] * x[i, a]
    return out


def gated_group_norm(y: torch.Tensor, z: torch.Tensor, weight: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    """``y silu(z)``, each of ``groups`` equal parts of a row divided by its own root mean square, times ``weight``."""
    n = y.shape[0]
    return over_rms((y * silu(z)).reshape(n, groups, -1), eps).reshape(n, -1) * weight


def state_space_mixer(h: torch.Tensor, t: Tensors, p: str, c: dict, eps: float) -> torch.Tensor:
    n, heads, vdim, size, groups = h.shape[0], c["heads"], c["vdim"], c["state"], c["groups"]
    inner, gn = heads * vdim, groups * size
    z, xbc, step = torch.split(h @ t[p + "in"].T, [inner, inner + 2 * gn, heads], dim=-1)
    xbc = silu(causal_conv(xbc, t[p + "conv"]) + t[p + "conv.b"])
    x, b, out = torch.split(xbc, [inner, gn, gn], dim=-1)
    step = torch.log1p(torch.exp(-(step + t[p + "dt_bias"]).abs())) + (step + t[p + "dt_bias"]).clamp(min=0)  # softplus
    y = state_space_scan(x.reshape(n, heads, vdim), b.reshape(n, groups, size), out.reshape(n, groups, size), step, torch.exp(t[p + "A_log"]), t[p + "D"])
    return gated_group_norm(y.reshape(n, inner), z, t[p + "norm"], c["norm_groups"], eps) @ t[p + "o"].T


def parallel_mixer(h: torch.Tensor, t: Tensors, p: str, c: dict, eps: float) -> torch.Tensor:
    left = kept_window_attention(h, t, p + "left.", c["left"], eps)
    right = state_space_mixer(h, t, p + "right.", c["right"], eps)
    return 0.5 * (rms_norm(left, t[p + "left.out"], eps) + rms_norm(right, t[p + "right.out"], eps))


MIXERS = {"attention": capped_attention_mixer, "parallel": parallel_mixer}


def feed_forward(h: torch.Tensor, t: Tensors, p: str) -> torch.Tensor:
    return (torch.relu(h @ t[p + "gate"].T) * (h @ t[p + "up"].T)) @ t[p + "down"].T


# ----------------------------------------------------------------------------------------------------------------------
# the model
# ----------------------------------------------------------------------------------------------------------------------
def run_order(config: dict) -> List[tuple]:
    """(layer, whether a pass of the loop begins with it) in the order of the runs."""
    count, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, False) for i in range(count)]
    start, stop = loop["start"], loop["stop"]
    order = [(i, False) for i in range(start)]
    for _ in range(loop["times"]):
        order += [(i, i == start) for i in range(start, stop)]
    return order + [(i, False) for i in range(stop, count)]


def forward(config: dict, tensors: Tensors, tokens: List[int], layer_outputs: Optional[list] = None) -> torch.Tensor:
    """Logits ``[n, vocab]`` of a whole sequence; ``layer_outputs`` gets the residual stream after every layer run."""
    eps = config["norm"]["eps"]
    start = tensors["embed"][torch.tensor(tokens, dtype=torch.long)]
    x = start
    for index, begins_pass in run_order(config):
        layer, p = config["layers"][index], f"l{index}."
        if begins_pass:
            x = torch.cat([x, start], dim=-1) @ tensors["loop.in"].T
        h = rms_norm(x, tensors[p + "norm1"], eps)
        y = MIXERS[layer["type"]](h, tensors, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            y = y + feed_forward(h, tensors, p + "mlp.")
        x = x + y
        if layer_outputs is not None:
            layer_outputs.append(x.clone())
    logits = rms_norm(x, tensors["final.norm"], eps) @ tensors["embed"].T
    return soft_cap(logits, config["logit_softcap"]) if config.get("logit_softcap") else logits


def read_folder(path):
    """-> (configuration, float64 tensors)."""
    from safetensors.torch import load_file

    with open(os.path.join(path, "config.json"), "r", encoding="utf-8") as handle:
        config = json.load(handle)
    return config, {name: t.double() for name, t in load_file(os.path.join(path, "model.safetensors")).items()}
