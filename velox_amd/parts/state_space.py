"""A selective state space with one decay per head (Mamba-2's recurrence).

Per head, with a state ``S`` of ``state x vdim`` float32 numbers, a step size ``d_t``, an input ``x_t`` of ``vdim`` channels and
vectors ``B_t`` and ``C_t`` of ``state`` entries that the heads of a group share (head ``h`` reads group ``h // (heads / groups)``):

    ``S <- exp(-exp(A_log_h) d_t) S + d_t B_t x_t^T``;   ``y_t = S^T C_t + D_h x_t``   with ``d_t = softplus(dt_t + dt_bias_h)``.

One product gives the row ``[z; x; B; C; dt]``.  x, B and C pass a short causal convolution per channel with a bias and SiLU; its
last ``taps - 1`` inputs are part of a sequence's state.  The read-out is multiplied by ``silu(z)`` and then normed in
``norm_groups`` equal parts, each by its own root mean square, with a weight per channel; then the output product.

Step sizes, decays, the state, the read-out, ``silu(z)`` on it and the norm are float32 in both run dtypes; the projections and the
convolution with its SiLU are the run dtype's.  The state lives in the request's state slot, ``[heads, state, vdim]`` float32,
beside the convolution's last inputs ``[taps - 1, channels]`` in the run dtype.

Kernels of a step: the product, the convolution, ``state_space_scan`` (step sizes, decays, recurrence, ``D``; token by token for
short portions, chunks on the float32 matrix instructions for long ones), ``gated_group_norm``, the output product.
"""
from __future__ import annotations

from typing import Dict, Optional, Tuple

import torch

from .base import Mixer, Param, StateNeed, register_part, single


class StateSpaceMixer(Mixer):
    def __init__(self, prefix: str, hidden_size: int, num_heads: int, groups: int, state: int, vdim: int, conv_taps: int, norm_groups: int,
                 norm_eps: float, names: Tuple[Tuple[str, str], ...] = ()) -> None:
        """``names``: pairs (tensor, name below the prefix) that replace the default names ``in``, ``conv``, ``conv.b``,
        ``dt_bias``, ``A_log``, ``D``, ``norm``, ``o``."""
        super().__init__(prefix)
        if min(int(num_heads), int(groups), int(state), int(vdim), int(conv_taps), int(norm_groups)) < 1 or not float(norm_eps) > 0:
            raise ValueError("heads, groups, state, vdim, conv_taps, norm_groups and norm_eps must be positive")
        if num_heads % groups != 0:
            raise ValueError(f"num_heads={num_heads} must be a multiple of groups={groups}")
        if num_heads * vdim % norm_groups != 0:
            raise ValueError(f"{num_heads * vdim} channels do not fall into {norm_groups} equal parts")
        self.hidden_size = int(hidden_size)
        self.num_heads, self.groups, self.state, self.vdim = int(num_heads), int(groups), int(state), int(vdim)
        self.conv_taps, self.norm_groups, self.norm_eps = int(conv_taps), int(norm_groups), float(norm_eps)
        self.names = {n: n for n in ("in", "conv", "conv.b", "dt_bias", "A_log", "D", "norm", "o")}
        self.names.update(dict(names))
        self.inner = self.num_heads * self.vdim
        self.conv_channels = self.inner + 2 * self.groups * self.state
        # columns of the first product: z, then what is convolved (x, B, C), then the step sizes
        self.conv_at, self.step_at = self.inner, self.inner + self.conv_channels
        self.in_weight = self.conv_weight = self.conv_bias = self.dt_bias = self.A_log = self.skip = self.norm_weight = self.o_weight = None
        self.rate: Optional[torch.Tensor] = None  # float32 [heads], exp(A_log)

    def params(self) -> Dict[str, Param]:
        h, n = self.hidden_size, self.names
        return {
            "in_weight": single(n["in"], (self.step_at + self.num_heads, h)),
            "conv_weight": single(n["conv"], (self.conv_channels, self.conv_taps), role="vector"),
            "conv_bias": single(n["conv.b"], (self.conv_channels,), role="vector"),
            "dt_bias": single(n["dt_bias"], (self.num_heads,), role="vector"),
            "A_log": single(n["A_log"], (self.num_heads,), role="vector"),
            "skip": single(n["D"], (self.num_heads,), role="vector", init="one_plus_normal"),
            "norm_weight": single(n["norm"], (self.inner,), role="vector", init="one_plus_normal"),
            "o_weight": single(n["o"], (h, self.inner)),
        }

    def cache_need(self):
        tensors = [("state", (self.num_heads, self.state, self.vdim), torch.float32)]
        if self.conv_taps >= 2:
            tensors.append(("conv_tail", (self.conv_taps - 1, self.conv_channels), None))
        return StateNeed(tuple(tensors))

    def finalize(self, device, dtype) -> None:
        self.refresh_derived()

    def refresh_derived(self) -> None:
        """The decay's rate per head; to be called again after a tensor was bound anew."""
        if self.A_log is not None:
            self.rate = torch.exp(self.A_log.float())

    def prepare_kernels(self, ops) -> None:
        self.prepare_weight(ops, "in_weight")
        self.prepare_weight(ops, "o_weight")
        check = getattr(ops, "state_space_supports", None)
        if check is not None:
            check(self.state, self.vdim)

    def forward(self, x, ctx, cache, owns_cache: bool = True):
        if not owns_cache:
            raise RuntimeError("a recurrent mixer cannot read another entry's state: every run of it advances a state of its own")
        ops = ctx.ops
        main = ops.linear(x, self.operand("in_weight"), None, ctx.dtype)
        tail = cache.tensors["conv_tail"] if self.conv_taps >= 2 else None
        xbc = ops.short_conv(main, self.conv_channels, self.conv_weight, tail, ctx.slots, ctx.cu_q, ctx.max_q_len, activation="silu",
                             first=self.conv_at, bias=self.conv_bias)
        read = ops.state_space_scan(xbc, main, self.step_at, self.dt_bias, self.rate, self.skip, cache.tensors["state"], ctx.slots, ctx.cu_q, ctx.max_q_len,
                                    self.num_heads, self.groups, self.state, self.vdim)
        y = ops.gated_group_norm(read, main, 0, self.norm_weight, self.norm_eps, self.norm_groups, ctx.dtype)
        return ops.linear(y, self.operand("o_weight"), None, ctx.dtype, partials_ok=True)


register_part("mixer", "state_space", StateSpaceMixer)
