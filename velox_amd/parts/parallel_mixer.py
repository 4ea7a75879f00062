"""Two mixers side by side: both read the same input, the result is ``left_scale * left(x) + right_scale * right(x)``, or,
with ``output_norm``, ``left_scale * norm_l(left(x)) + right_scale * norm_r(right(x))`` with a norm of its own behind each.

The two are parts of any registered mixer kinds, built from their ``PartSpec`` under ``<prefix><left_prefix>`` and
``<prefix><right_prefix>``; each keeps the cache or state its own kind asks for (the pair's need is the
``CompositeNeed`` of theirs).  The weighted sum is not a pass of its own: it is handed on as a ``ScaledSum`` (with norms: a
``NormedSum``), which the kernel that adds a sub-layer's output to the residual forms in float32.
"""
from __future__ import annotations

from typing import Optional, Tuple

from .base import CompositeNeed, Mixer, NormedSum, Part, PartSpec, ScaledSum, make_part, register_part


class ParallelMixer(Mixer):
    def __init__(self, prefix: str, left: PartSpec, right: PartSpec, left_scale: float = 1.0, right_scale: float = 1.0,
                 left_prefix: str = "left.", right_prefix: str = "right.", position=None, position_to: Tuple[bool, bool] = (True, False),
                 output_norm: Optional[PartSpec] = None, output_norm_prefixes: Tuple[str, str] = ("left.out", "right.out")) -> None:
        """``position``: the layer's position encoding (a part); ``position_to`` says which of the two mixers takes it.
        ``output_norm``: the kind and constants of the norms behind the two mixers (a kind with a ``deferred_form``), whose
        tensors stand under the mixer's prefix and ``output_norm_prefixes``."""
        super().__init__(prefix)
        self.scales = (float(left_scale), float(right_scale))
        self.mixers = []
        for spec, below, takes in ((left, left_prefix, position_to[0]), (right, right_prefix, position_to[1])):
            kwargs = spec.kwargs()
            if position is not None and takes:
                kwargs["position"] = position
            self.mixers.append(make_part("mixer", spec.kind, prefix=prefix + below, **kwargs))

        self.output_norms = ()
        if output_norm is not None:
            self.output_norms = tuple(make_part("norm", output_norm.kind, prefix=prefix + below, **output_norm.kwargs()) for below in output_norm_prefixes)

    def children(self) -> Tuple[Part, ...]:
        return (*self.mixers, *self.output_norms)

    def cache_need(self):
        return CompositeNeed(tuple(mixer.cache_need() for mixer in self.mixers))

    def forward(self, x, ctx, cache, owns_cache: bool = True):
        outputs = [mixer.forward(x, ctx, view, owns_cache) for mixer, view in zip(self.mixers, cache.views)]
        if self.output_norms:
            forms = [norm.deferred_form() for norm in self.output_norms]
            return NormedSum(tuple(outputs), tuple(form[0] for form in forms), self.scales, forms[0][1])
        outputs = [y.sum(0) if y.dim() == 3 else y for y in outputs]
        return ScaledSum(tuple(outputs), self.scales)


register_part("mixer", "parallel_mixers", ParallelMixer)
