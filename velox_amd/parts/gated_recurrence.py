"""Recurrences that work on every channel by itself: ``S_t = (1 - z_t) S_(t-1) + z_t c_t``, with gates that do not
depend on the state (a minimal gated recurrent unit).

``z = sigmoid(W_z x + b_z)`` and ``u = W_x x + b_x``, both of ``width`` channels; the candidate ``c`` is ``u + shift`` where ``u >= 0`` and
``sigmoid(u)`` where ``u < 0`` (continuous at 0 for a shift of 1/2, and positive everywhere); the output is
``W_o (S * silu(W_g x))``.  Because the gates do not read the state, the recurrence is linear in it and a portion of a prompt can be
cut into pieces that are worked at the same time: ``S`` behind a piece is ``A S_before + B`` with ``A`` the product of the piece's
``1 - z`` and ``B`` its own state from zero.

Gates, candidate and state are float32; the state, ``[width]``, lives in the request's state slot.  Kernels of a step: one
product ``[z; x; g]``, ``gated_scan`` (biases, gates, recurrence and output gate; two passes over pieces for longer portions),
the output product.
"""
from __future__ import annotations

from typing import Dict, Tuple

import torch

from .base import Mixer, Param, StateNeed, fused_rows, register_part, single


class GatedRecurrenceMixer(Mixer):
    def __init__(self, prefix: str, hidden_size: int, width: int, shift: float = 0.5, names: Tuple[Tuple[str, str], ...] = ()) -> None:
        """``names``: pairs (tensor, name below the prefix) that replace the default names; a bias is the tensor's name with
        ``.b`` added."""
        super().__init__(prefix)
        if int(width) < 1:
            raise ValueError(f"width={width} must be positive")
        self.hidden_size = int(hidden_size)
        self.width = int(width)
        self.shift = float(shift)
        self.names = {"z": "z", "x": "x", "g": "g", "o": "o"}
        self.names.update(dict(names))
        self.in_weight = self.gate_bias = self.input_bias = self.o_weight = None

    def params(self) -> Dict[str, Param]:
        h, w, n = self.hidden_size, self.width, self.names
        return {
            "in_weight": fused_rows((n["z"], n["x"], n["g"]), ((w, h),) * 3),
            "gate_bias": single(n["z"] + ".b", (w,), role="vector"),
            "input_bias": single(n["x"] + ".b", (w,), role="vector"),
            "o_weight": single(n["o"], (h, w)),
        }

    def cache_need(self):
        return StateNeed((("state", (self.width,), torch.float32),))

    def prepare_kernels(self, ops) -> None:
        self.prepare_weight(ops, "in_weight")
        self.prepare_weight(ops, "o_weight")

    def forward(self, x, ctx, cache, owns_cache: bool = True):
        if not owns_cache:
            raise RuntimeError("a recurrent mixer cannot read another entry's state: every run of it advances a state of its own")
        ops = ctx.ops
        projected = ops.linear(x, self.operand("in_weight"), None, ctx.dtype)
        y = ops.gated_scan(projected, self.width, self.gate_bias, self.input_bias, self.shift, cache.tensors["state"], ctx.slots, ctx.cu_q, ctx.max_q_len)
        return ops.linear(y, self.operand("o_weight"), None, ctx.dtype, partials_ok=True)


register_part("mixer", "gated_recurrence", GatedRecurrenceMixer)
