"""Kedanex, written out plainly: whole sequences, no cache, token-by-token loops, one function per mechanism.

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


def unit_vector(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def rotate_halves(x: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """``x`` [n, heads, d]: channel ``i`` of the first ``dims`` is turned with channel ``i + dims / 2``; the rest passes."""
    half = dims // 2
    freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64)
    angle = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * freq[None, :]
    cos, sin = angle.cos().to(x.dtype)[:, None, :], angle.sin().to(x.dtype)[:, None, :]
    first, second = x[..., :half], x[..., half:dims]
    return torch.cat([first * cos - second * sin, second * cos + first * sin, x[..., dims:]], dim=-1)


def softmax_with_silent_key(scores: torch.Tensor) -> torch.Tensor:
    """``exp(s_j) / (1 + sum exp(s))``: a softmax with one more key, of score 0, that has no value."""
    top = torch.clamp(scores.max(), min=0.0)
    weights = torch.exp(scores - top)
    return weights / (torch.exp(-top) + weights.sum())


# ----------------------------------------------------------------------------------------------------------------------
# mixers
# ----------------------------------------------------------------------------------------------------------------------
def general_delta_decay(h: torch.Tensor, t: Tensors, p: str) -> torch.Tensor:
    """``exp(-e^(-1/2) sigmoid(W_w2 tanh(W_w1 h) + w0))``, [n, heads * dim]."""
    z = torch.tanh(h @ t[p + "w1"].T) @ t[p + "w2"].T + t[p + "w0"]
    return torch.exp(-math.exp(-0.5) * torch.sigmoid(z))


def general_delta_scan(r, k, v, decay, removal) -> torch.Tensor:
    """All [n, heads, d].  Per head ``S <- diag(decay) S - (removal * u) (u^T S) + k v^T`` with ``u`` the unit vector of ``k``,
    both terms on the old state; ``o = S^T r`` on the new one."""
    n, heads, d = r.shape
    out = torch.zeros_like(v)
    for a in range(heads):
        state = torch.zeros(d, d, dtype=r.dtype)
        for i in range(n):
            u = unit_vector(k[i, a])
            state = decay[i, a][:, None] * state - torch.outer(removal[i, a] * u, u @ state) + torch.outer(k[i, a], v[i, a])
            out[i, a] = state.T @ r[i, a]
    return out


def general_delta_mixer(h: torch.Tensor, t: Tensors, p: str, c: dict, eps: float) -> torch.Tensor:
    n, heads, dim = h.shape[0], c["heads"], c["dim"]

    def per_head(y):
        return y.reshape(n, heads, dim)

    r, k, v = (per_head(h @ t[p + name].T) for name in ("r", "k", "v"))
    removal = per_head(torch.sigmoid(h @ t[p + "a"].T + t[p + "a.b"]))
    o = general_delta_scan(r, k, v, per_head(general_delta_decay(h, t, p)), removal)
    o = over_rms(o, eps).reshape(n, heads * dim) * t[p + "norm"] * torch.sigmoid(h @ t[p + "g"].T)
    return o @ t[p + "o"].T


def mingru_mixer(h: torch.Tensor, t: Tensors, p: str, c: dict, eps: float) -> torch.Tensor:
    z = torch.sigmoid(h @ t[p + "z"].T + t[p + "z.b"])
    u = h @ t[p + "x"].T + t[p + "x.b"]
    candidate = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    state = torch.zeros(c["width"], dtype=h.dtype)
    states = torch.zeros(h.shape[0], c["width"], dtype=h.dtype)
    for i in range(h.shape[0]):
        state = (1.0 - z[i]) * state + z[i] * candidate[i]
        states[i] = state
    return (states * silu(h @ t[p + "g"].T)) @ t[p + "o"].T


def window_attention_mixer(h: torch.Tensor, t: Tensors, p: str, c: dict, eps: float) -> torch.Tensor:
    n, heads, groups, dim = h.shape[0], c["heads"], c["kv_heads"], c["dim"]
    q = (h @ t[p + "q"].T).reshape(n, heads, dim)
    k = (h @ t[p + "k"].T).reshape(n, groups, dim)
    v = k
    if c.get("rot"):
        q, k = rotate_halves(q, c["rot"]["dims"], c["rot"]["base"]), rotate_halves(k, c["rot"]["dims"], c["rot"]["base"])
    q, k = over_rms(q, eps), over_rms(k, eps)
    window = (c.get("mask") or {}).get("size")
    out = torch.zeros(n, heads, dim, dtype=h.dtype)
    for i in range(n):
        lo = 0 if window is None else max(0, i - window + 1)
        for a in range(heads):
            g = a // (heads // groups)
            weights = softmax_with_silent_key((k[lo:i + 1, g] @ q[i, a]) * c["scale"])
            out[i, a] = weights @ v[lo:i + 1, g]
    return out.reshape(n, heads * dim) @ t[p + "o"].T


MIXERS = {"general_delta": general_delta_mixer, "mingru": mingru_mixer, "attention": window_attention_mixer}


# ----------------------------------------------------------------------------------------------------------------------
# feed-forwards
# ----------------------------------------------------------------------------------------------------------------------
def poly_norm(z: torch.Tensor, coefficients: torch.Tensor, eps: float) -> torch.Tensor:
    """``a N(z) + b N(z^2) + c N(z^3) + e``; ``N`` divides a row by its root mean square."""
    a, b, c, e = coefficients
    return a * over_rms(z, eps) + b * over_rms(z ** 2, eps) + c * over_rms(z ** 3, eps) + e


def dense_feed_forward(h: torch.Tensor, t: Tensors, p: str, eps: float) -> torch.Tensor:
    return poly_norm(h @ t[p + "up"].T, t[p + "act"], eps) @ t[p + "down"].T


def choose_experts(logits: torch.Tensor, top: int):
    """-> (expert index [n, top], weight [n, top]): the largest logits, softmax over the chosen ones."""
    values, index = logits.topk(top, dim=-1)
    return index, torch.softmax(values, dim=-1)


def mixture_feed_forward(h: torch.Tensor, t: Tensors, p: str, c: dict) -> torch.Tensor:
    index, weight = choose_experts(h @ t[p + "router"].T, c["router"]["top"])
    out = torch.zeros_like(h)
    for i in range(h.shape[0]):
        for e, w in zip(index[i].tolist(), weight[i]):
            q = f"{p}e{e}."
            out[i] += w * (t[q + "down"] @ (silu(t[q + "gate"] @ h[i]) * (t[q + "up"] @ h[i])))
    return out


def feed_forward(mlp: dict, h: torch.Tensor, t: Tensors, p: str, eps: float) -> torch.Tensor:
    if mlp["kind"] == "dense":
        return dense_feed_forward(h, t, p, eps)
    return mixture_feed_forward(h, t, p, mlp)


# ----------------------------------------------------------------------------------------------------------------------
# the model
# ----------------------------------------------------------------------------------------------------------------------
def forward(config: dict, tensors: Tensors, tokens: List[int], layer_outputs: Optional[list] = None) -> torch.Tensor:
    """Logits ``[n, vocab]`` of a whole sequence; ``layer_outputs`` gets the residual stream after every layer run."""
    eps = config["norm"]["eps"]
    x = tensors["embed"][torch.tensor(tokens, dtype=torch.long)]
    for index, layer in enumerate(config["layers"]):
        owner = index
        while config["layers"][owner].get("weights_of") is not None:
            owner = config["layers"][owner]["weights_of"]
        p = f"l{owner}."
        y = MIXERS[layer["type"]](rms_norm(x, tensors[p + "norm1"], eps), tensors, p + "mix.", layer["mixer"], eps)
        x = x + rms_norm(y, tensors[p + "norm1b"], eps)
        if layer.get("mlp") is not None:
            y = feed_forward(layer["mlp"], rms_norm(x, tensors[p + "norm2"], eps), tensors, p + "mlp.", eps)
            x = x + rms_norm(y, tensors[p + "norm2b"], eps)
        if layer_outputs is not None:
            layer_outputs.append(x.clone())
    return rms_norm(x, tensors["final.norm"], eps) @ tensors["head"].T


def read_folder(path):
    """-> (configuration, float64 tensors)."""
    from safetensors.torch import load_file

    with open(os.path.join(path, "config.json"), "r", encoding="utf-8") as handle:
        config = json.load(handle)
    return config, {name: t.double() for name, t in load_file(os.path.join(path, "model.safetensors")).items()}
