"""A decoder described as data, and the object built from that description.

``ModelSpec`` is what an architecture produces from its configuration: one
``LayerSpec`` per weight-owning layer (each naming its own mixer, feed-forward and
norm kinds with their constants), shared position encodings, and ``schedule``, the
order in which layers run.  The schedule is a list of ``ScheduleEntry``: an entry may
name a layer that an earlier entry already named (the layer's weights run twice, each
run with a cache of its own), begin a pass of a loop over layers (``begins_pass``: the
model's ``pass_input`` then makes that pass's residual first), or set ``cache_from`` to an earlier entry to read that
entry's cache instead of owning one.

``DecoderModel`` runs the whole thing the way the reference's ``QwenDecoderModel``
does (``src/transformer.py:43-52``): embed, blocks in schedule order, final norm; the
output head is a separate call on chosen rows (``src/transformer.py:67-68``).
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple

import torch

from . import block as _block  # noqa: F401  (registers the built-in arrangement)
from .base import Embedding, OutputHead, Param, Part, PartSpec, PassInput, StateNeed, make_part, register_part, single


@dataclass(frozen=True)
class LayerSpec:
    prefix: str
    mixer: PartSpec
    feed_forward: PartSpec
    mixer_norm: PartSpec
    ff_norm: PartSpec
    position: Optional[str] = None  # key into ModelSpec.positions handed to the mixer
    arrangement: str = "pre_norm"
    arrangement_args: Tuple[Tuple[str, object], ...] = ()  # constants of the arrangement (sorted pairs, as in PartSpec)
    # where each part's tensors stand in the checkpoint, below the layer's prefix (an architecture sets its own names)
    mixer_prefix: str = "mixer."
    feed_forward_prefix: str = "feed_forward."
    mixer_norm_prefix: str = "mixer_norm."
    ff_norm_prefix: str = "feed_forward_norm."


@dataclass(frozen=True)
class ScheduleEntry:
    layer: int
    cache_from: Optional[int] = None
    begins_pass: bool = False


@dataclass
class ModelSpec:
    vocab_size: int
    hidden_size: int
    max_position: int
    layers: List[LayerSpec]
    schedule: List[ScheduleEntry]
    final_norm: PartSpec
    positions: Dict[str, PartSpec] = field(default_factory=dict)
    embedding_position: Optional[str] = None  # a position encoding applied to the embeddings
    tie_head: bool = False
    embed_name: str = "embedding.weight"
    head_name: str = "head.weight"
    final_norm_prefix: str = "final_norm."
    eos_token_ids: Tuple[int, ...] = ()
    # The parts at the two ends, chosen like every other part.  None = the plain ones: a table that is looked up
    # (``embed_name``) and a product without bias (``head_name``, or the table itself with ``tie_head``).  A kind
    # registered under "embedding" / "head" gets its ``args`` plus ``name``, ``vocab_size``, ``hidden_size`` and, for a
    # head, ``tied_to`` (the table's checkpoint name or None).
    embedding: Optional[PartSpec] = None
    head: Optional[PartSpec] = None
    # Copies of the residual that the blocks keep side by side (hyper-connections): the residual is then float32
    # ``[T, residual_streams * H]``, every copy starts as the embedding output, and the final norm reads their sum.
    residual_streams: int = 1
    # What makes the residual of every schedule entry that begins a pass (a kind registered under "pass_input"; it gets
    # its ``args`` plus ``hidden_size``).
    pass_input: Optional[PartSpec] = None

    def validate(self) -> None:
        if not self.layers:
            raise ValueError("a model needs at least one layer")
        for index, entry in enumerate(self.schedule):
            if not 0 <= entry.layer < len(self.layers):
                raise ValueError(f"schedule[{index}] names layer {entry.layer}, but there are {len(self.layers)}")
            if entry.cache_from is not None:
                if not 0 <= entry.cache_from < index:
                    raise ValueError(f"schedule[{index}].cache_from must name an earlier entry")
                if self.schedule[entry.cache_from].cache_from is not None:
                    raise ValueError(f"schedule[{index}].cache_from must name an entry that owns its cache")
            if entry.begins_pass and (self.pass_input is None or self.residual_streams != 1):
                raise ValueError(f"schedule[{index}] begins a pass: the model needs a pass_input, and one residual stream")


class TableEmbedding(Embedding):
    """``h[t] = E[ids[t]] * scale``; the reference has no scaling (``src/transformer.py:27,44``), which is ``scale`` = 1.
    The product is taken in float32, inside the kernel that looks the rows up."""

    def __init__(self, name: str, vocab_size: int, hidden_size: int, scale: float = 1.0) -> None:
        super().__init__("")
        self.name = name
        self.vocab_size = vocab_size
        self.hidden_size = hidden_size
        self.scale = float(scale)
        self.table: Optional[torch.Tensor] = None

    def params(self) -> Dict[str, Param]:
        return {"table": single(self.name, (self.vocab_size, self.hidden_size), product=False)}

    def forward(self, token_ids: torch.Tensor, ctx, copies: int = 1) -> torch.Tensor:
        """``copies`` > 1: the row is written that many times side by side, ``[T, copies * H]``."""
        if copies != 1:
            return ctx.ops.embed(token_ids, self.table, scale=self.scale, copies=copies)
        if self.scale == 1.0:
            return ctx.ops.embed(token_ids, self.table)
        return ctx.ops.embed(token_ids, self.table, scale=self.scale)


class BigramEmbedding(TableEmbedding):
    """``h[t] = E[ids[t]] * scale + B[(ids[t-1] * mul_prev + ids[t] * mul_cur) mod buckets]``: beside the token's own row, a
    row of a second table chosen by a hash of the token and the one before it; a sequence's first token reads the
    table's last row (row ``buckets``).  The token before a portion's first one is part of the request's state: one
    int32 per state slot, which the kernel that looks the rows up reads for a portion's first token and sets to the
    portion's last token (a request at position 0 does not read it).  The sum is float32."""

    def __init__(self, name: str, vocab_size: int, hidden_size: int, buckets: int, mul_prev: int, mul_cur: int, scale: float = 1.0,
                 bigram_name: str = "bigram") -> None:
        super().__init__(name, vocab_size, hidden_size, scale)
        if int(buckets) < 1:
            raise ValueError(f"buckets={buckets} must be positive")
        self.buckets, self.mul_prev, self.mul_cur = int(buckets), int(mul_prev), int(mul_cur)
        self.bigram_name = bigram_name
        self.bigram: Optional[torch.Tensor] = None

    def params(self) -> Dict[str, Param]:
        out = super().params()
        out["bigram"] = single(self.bigram_name, (self.buckets + 1, self.hidden_size), product=False)
        return out

    def cache_need(self):
        return StateNeed((("previous_token", (1,), torch.int32),))

    def forward(self, token_ids: torch.Tensor, ctx, copies: int = 1, cache=None) -> torch.Tensor:
        if copies != 1:
            raise ValueError("the bigram embedding writes one residual stream")
        if cache is None:
            raise ValueError("the bigram embedding needs its state (the token before each portion)")
        return ctx.ops.embed_bigram(token_ids, self.table, self.bigram, self.scale, self.buckets, self.mul_prev, self.mul_cur,
                                    ctx.positions, ctx.cu_q, ctx.slots, cache.tensors["previous_token"], ctx.max_q_len)


class LinearPassInput(PassInput):
    """``x <- W [x; start]``: the residual and the embedding output side by side through one product without bias, whose
    float32 result is the pass's residual.  The kernel that adds what is pending writes both halves of the product's
    input and clears the residual, so the product is what the next norm adds, like any sub-layer's output."""

    def __init__(self, hidden_size: int, name: str = "pass.in") -> None:
        super().__init__("")
        self.hidden_size = int(hidden_size)
        self.name = name
        self.weight: Optional[torch.Tensor] = None

    def params(self) -> Dict[str, Param]:
        return {"weight": single(self.name, (self.hidden_size, 2 * self.hidden_size))}

    def prepare_kernels(self, ops) -> None:
        self.prepare_weight(ops, "weight")

    def forward(self, residual, pending, start, ctx):
        joined = ctx.ops.join_rows(residual, pending, start, ctx.dtype)
        return ctx.ops.linear(joined, self.operand("weight"), None, torch.float32, partials_ok=True)


class LinearHead(OutputHead):
    """``logits = (hidden @ W^T) * scale`` without bias; ``W`` is the embedding table when tied
    (reference ``src/transformer.py:60-62``; it has no scale, which is ``scale`` = 1), then ``cap * tanh(logits / cap)`` with
    ``softcap``.  Logits are returned in float32 and both are applied to them there."""

    def __init__(self, name: str, vocab_size: int, hidden_size: int, tied_to: Optional[str] = None, scale: float = 1.0,
                 softcap: Optional[float] = None) -> None:
        super().__init__("")
        if softcap is not None and not float(softcap) > 0:
            raise ValueError(f"softcap={softcap} must be positive")
        self.scale = float(scale)
        self.softcap = float(softcap) if softcap is not None else None
        self.name = name
        self.vocab_size = vocab_size
        self.hidden_size = hidden_size
        self.tied_to = tied_to
        self.weight: Optional[torch.Tensor] = None

    def params(self) -> Dict[str, Param]:
        base = single(self.name, (self.vocab_size, self.hidden_size))
        if self.tied_to is None:
            return {"weight": base}
        return {"weight": Param(base.shape, base.sources, base.source_shapes, base.role, base.init, alias_of=self.tied_to)}

    def prepare_kernels(self, ops) -> None:
        self.prepare_weight(ops, "weight")

    def forward(self, hidden_rows: torch.Tensor, ctx) -> torch.Tensor:
        logits = ctx.ops.linear(hidden_rows, self.operand("weight"), None, torch.float32)
        if self.softcap is not None:
            return ctx.ops.softcap_(logits, self.softcap, self.scale)
        return logits if self.scale == 1.0 else ctx.ops.scale_(logits, self.scale)


register_part("embedding", "table", TableEmbedding)
register_part("embedding", "bigram_table", BigramEmbedding)
register_part("head", "linear", LinearHead)
register_part("pass_input", "linear", LinearPassInput)

EMBEDDING_OUTPUT = "embedding_output"  # key in a step's shared values: the embedding output, for models whose passes read it


class DecoderModel(Part):
    def __init__(self, spec: ModelSpec) -> None:
        super().__init__("")
        spec.validate()
        self.spec = spec
        self.positions = {key: make_part("position", ps.kind, **ps.kwargs()) for key, ps in spec.positions.items()}
        embedding = spec.embedding or PartSpec.of("table")
        self.embedding = make_part("embedding", embedding.kind, name=spec.embed_name, vocab_size=spec.vocab_size, hidden_size=spec.hidden_size, **embedding.kwargs())
        self.blocks = []
        for layer in spec.layers:
            mixer_kwargs = layer.mixer.kwargs()
            if layer.position is not None:
                mixer_kwargs["position"] = self.positions[layer.position]
            mixer = make_part("mixer", layer.mixer.kind, prefix=layer.prefix + layer.mixer_prefix, **mixer_kwargs)
            ff = make_part("feed_forward", layer.feed_forward.kind, prefix=layer.prefix + layer.feed_forward_prefix, **layer.feed_forward.kwargs())
            norm1 = make_part("norm", layer.mixer_norm.kind, prefix=layer.prefix + layer.mixer_norm_prefix, **layer.mixer_norm.kwargs())
            norm2 = make_part("norm", layer.ff_norm.kind, prefix=layer.prefix + layer.ff_norm_prefix, **layer.ff_norm.kwargs())
            self.blocks.append(make_part("arrangement", layer.arrangement, prefix=layer.prefix, mixer=mixer, feed_forward=ff, mixer_norm=norm1, ff_norm=norm2,
                                         **dict(layer.arrangement_args)))
        self.final_norm = make_part("norm", spec.final_norm.kind, prefix=spec.final_norm_prefix, **spec.final_norm.kwargs())
        head = spec.head or PartSpec.of("linear")
        self.head = make_part("head", head.kind, name=spec.head_name, vocab_size=spec.vocab_size, hidden_size=spec.hidden_size,
                              tied_to=spec.embed_name if spec.tie_head else None, **head.kwargs())
        self.pass_input = make_part("pass_input", spec.pass_input.kind, hidden_size=spec.hidden_size, **spec.pass_input.kwargs()) if spec.pass_input is not None else None
        self.schedule = list(spec.schedule)

    # -- structure ----------------------------------------------------------------------
    def children(self) -> Tuple[Part, ...]:
        joint = (self.pass_input,) if self.pass_input is not None else ()
        return (self.embedding, *self.positions.values(), *joint, *self.blocks, self.final_norm, self.head)

    def all_parts(self) -> List[Part]:
        out: List[Part] = []

        def walk(part: Part) -> None:
            out.append(part)
            for child in part.children():
                walk(child)

        for child in self.children():
            walk(child)
        return out

    def allows_capture(self) -> bool:
        """Whether every part allows its ``forward`` to be captured into a HIP graph (``Part.graph_safe``)."""
        return all(part.graph_safe for part in self.all_parts())

    def cache_needs(self) -> List[object]:
        """One entry per schedule entry: the mixer's need, or None when it reads another entry's cache.  An embedding
        that keeps something per request (``Embedding.cache_need``) adds one entry behind the schedule's."""
        needs = []
        for entry in self.schedule:
            need = self.blocks[entry.layer].cache_need()
            needs.append(need if entry.cache_from is None else None)
        if self.embedding.cache_need() is not None:
            needs.append(self.embedding.cache_need())
        return needs

    # -- arithmetic ---------------------------------------------------------------------
    def embed(self, token_ids: torch.Tensor, ctx) -> torch.Tensor:
        """The residual stream before the first block: float32 ``[T, H]``."""
        streams = self.spec.residual_streams
        if self.embedding.cache_need() is not None:
            residual = self.embedding.forward(token_ids, ctx, cache=ctx.cache_view(len(self.schedule)))
            if self.spec.embedding_position is not None:
                residual = self.positions[self.spec.embedding_position].on_embeddings(residual, ctx)
            return residual.repeat(1, streams) if streams > 1 else residual
        if streams > 1 and self.spec.embedding_position is None:
            return self.embedding.forward(token_ids, ctx, copies=streams)  # (the looked-up row written once per stream)
        residual = self.embedding.forward(token_ids, ctx)
        if self.spec.embedding_position is not None:
            residual = self.positions[self.spec.embedding_position].on_embeddings(residual, ctx)
        return residual.repeat(1, streams) if streams > 1 else residual

    def begin(self, token_ids: torch.Tensor, ctx) -> torch.Tensor:
        """``embed``, with the embedding output kept for the passes that read it."""
        residual = self.embed(token_ids, ctx)
        if self.pass_input is not None:
            ctx.shared[EMBEDDING_OUTPUT] = ctx.ops.kept_copy(residual, ctx.dtype)  # (blocks update the residual in place)
        return residual

    def run_schedule(self, residual: torch.Tensor, pending, ctx, first: int = 0, last: Optional[int] = None):
        """Runs schedule entries ``first .. last - 1`` on ``residual`` (updated in place); takes and returns ``pending``,
        the sub-layer output that the next norm still has to add."""
        last = len(self.schedule) if last is None else last
        for index in range(first, last):
            entry = self.schedule[index]
            owner = index if entry.cache_from is None else entry.cache_from
            cache = ctx.cache_view(owner)
            # the norm that reads this block's output: the one the next entry's block begins with, if it begins with one
            # (the final norm works on chosen rows and takes its input as it is)
            following = self.blocks[self.schedule[index + 1].layer].input_norm() if index + 1 < len(self.schedule) and not self.schedule[index + 1].begins_pass else None
            if entry.begins_pass:
                pending = self.pass_input.forward(residual, pending, ctx.shared[EMBEDDING_OUTPUT], ctx)
            pending = self.blocks[entry.layer].forward(residual, pending, ctx, cache, entry.cache_from is None, next_norm=following)
        return pending

    def forward(self, token_ids: torch.Tensor, ctx):
        """Runs every block; returns ``(residual float32 [T, H], pending [T, H])``."""
        residual = self.begin(token_ids, ctx)
        return residual, self.run_schedule(residual, None, ctx)

    def logits(self, residual: torch.Tensor, pending, rows: torch.Tensor, ctx) -> torch.Tensor:
        """Final norm and output head on ``rows`` (int32 [R]) only: float32 [R, vocab]."""
        hidden = self.final_norm.forward(residual, pending, ctx, rows=rows)
        return self.head.forward(hidden, ctx)
