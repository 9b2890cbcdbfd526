"""A model: parts built from a layout, loaded from a tensor source, and run
entry by entry of the layout's order.

The reference's counterpart is the weight-only ``Transformer`` skeleton
(``fastgen/model.py:151-202``) plus the layer loop of ``_forward``
(``fastgen/forward.py:347-515``).
"""

from __future__ import annotations

import inspect
import math
from dataclasses import dataclass, field
from pathlib import Path
from typing import Any, Dict, List, Mapping, Optional, Sequence

import torch

from ..config import ModelLayout, PartSpec, get_architecture, read_config_json
from ..kernels.linear import StreamedMatrix, packing, packing_fits
from ..kernels.ops import (PostNormed, ScaledDelta, ScaledRows, StreamTerms, post_add_rmsnorm, stream_add, stream_terms,
                           streams_spread)
from ..parts import LayerStore, PagedNeed, StateNeed, TensorSpec, build_part
from ..parts.base import MATRIX
from ..weights.source import RandomSource, SafetensorsSource, TensorSource, check_against_specs
from .context import StepContext


@dataclass
class ModelParts:
    layout: ModelLayout
    embed: Any
    blocks: List[Any]
    mixers: List[Any]
    final_norm: Any
    head: Any
    all_parts: List[Any]
    injections: List[Any] = field(default_factory=list)

    def tensor_specs(self) -> List[TensorSpec]:
        return [s for p in self.all_parts for s in p.tensor_specs()]

    def duplicates(self) -> Mapping[str, str]:
        return dict(self.head.duplicates()) if hasattr(self.head, "duplicates") else {}


def build_parts(layout: ModelLayout) -> ModelParts:
    """Every part of the layout, looked up by kind; nothing is on a device yet."""
    embed = build_part("embedding", layout.embed)
    blocks, mixers, parts = [], [], [embed]
    for ls in layout.layers:
        mixer = build_part("mixer", ls.mixer)
        ffn = build_part("feed_forward", ls.ffn) if ls.ffn is not None else None
        n1 = build_part("norm", ls.mixer_norm)
        n2 = build_part("norm", ls.ffn_norm) if ls.ffn_norm is not None else None
        extra = {name: build_part("norm", spec) for name, spec in ls.extra_norms.items()}
        # an arrangement that asks for no further norms is built from the four parts alone
        block = build_part("arrangement", ls.arrangement_spec or PartSpec(ls.arrangement), mixer, ffn, n1, n2,
                           *([extra] if extra else []))
        blocks.append(block)
        mixers.append(mixer)
        parts += [p for p in (mixer, ffn, n1, n2, *extra.values()) if p is not None]
        if hasattr(block, "tensor_specs"):  # an arrangement with tensors of its own
            parts.append(block)
    injections = [build_part("injection", spec) for spec in layout.injections]
    final_norm = build_part("norm", layout.final_norm)
    head = build_part("head", layout.head)
    parts += [*injections, final_norm, head]
    return ModelParts(layout, embed, blocks, mixers, final_norm, head, parts, injections)


class Model:
    def __init__(self, layout: ModelLayout, dtype: torch.dtype, device: torch.device | str, args: Any = None,
                 architecture: Optional[str] = None, packed_weights: Optional[bool] = None,
                 memory_budget: Optional[int] = None) -> None:
        """``packed_weights``: whether the bfloat16 matrices get a second copy in the order in which the
        products of few rows read them (``kernels.linear.StreamedMatrix``); None: if the weights twice
        leave half of ``memory_budget`` (bytes for the model and its cache; default: the GPU's memory) free
        (``kernels.linear.packing_fits``)."""
        if dtype not in (torch.float32, torch.bfloat16):
            raise ValueError(f"dtype {dtype} is not supported (float32 or bfloat16)")
        self.layout, self.dtype, self.device = layout, dtype, torch.device(device)
        self.args, self.architecture = args, architecture
        self.packed_weights, self.memory_budget = packed_weights, memory_budget
        self.parts = build_parts(layout)
        self.vocab_size = layout.vocab_size
        self.loaded = False

    # ------------------------------------------------------------- build
    @classmethod
    def from_config(cls, config: Mapping[str, Any], dtype: torch.dtype, device: torch.device | str,
                    packed_weights: Optional[bool] = None, memory_budget: Optional[int] = None,
                    source: Optional[TensorSource] = None) -> "Model":
        """``source``: the checkpoint, for an architecture some of whose sizes only the tensors' shapes give
        (its ``parse`` then takes a second argument, a function from a tensor's name to its shape or None)."""
        arch = get_architecture(config)
        if source is not None and len(inspect.signature(arch.parse).parameters) > 1:
            names = set(source.names())
            args = arch.parse(config, lambda name: source.shape(name) if name in names else None)
        else:
            args = arch.parse(config)
        return cls(arch.layout(args), dtype, device, args=args, architecture=arch.name, packed_weights=packed_weights,
                   memory_budget=memory_budget)

    @classmethod
    def from_folder(cls, model_dir: str | Path, dtype: torch.dtype, device: torch.device | str,
                    packed_weights: Optional[bool] = None, memory_budget: Optional[int] = None) -> "Model":
        """The model that ``config.json`` names, with the folder's weights."""
        source = SafetensorsSource(model_dir)
        model = cls.from_config(read_config_json(model_dir), dtype, device, packed_weights, memory_budget, source)
        model.load(source)
        return model

    @classmethod
    def random(cls, config: Mapping[str, Any], seed: int, dtype: torch.dtype,
               device: torch.device | str, packed_weights: Optional[bool] = None,
               memory_budget: Optional[int] = None) -> "Model":
        """Seeded random weights drawn on the device, without a folder."""
        model = cls.from_config(config, dtype, device, packed_weights, memory_budget)
        model.load(RandomSource(model.parts.tensor_specs(), seed, dtype, device))
        return model

    def load(self, source: TensorSource) -> None:
        specs = self.parts.tensor_specs()
        check_against_specs(source, specs, self.parts.duplicates())
        pack = self.packed_weights
        if pack is None:
            matrix_bytes = sum(math.prod(s.shape) for s in specs if s.role == MATRIX) * 2
            pack = self.dtype == torch.bfloat16 and packing_fits(matrix_bytes, self.device, self.memory_budget)
        with packing(pack and self.dtype == torch.bfloat16):
            for part in self.parts.all_parts:
                tensors = {s.name: source.get(s.name) for s in part.tensor_specs()}
                part.load(tensors, self.dtype, self.device)
            if getattr(self.parts.head, "tied_to", None):
                self.parts.head.tie(self.parts.embed.weight)
        self.loaded = True

    # ------------------------------------------------------------- needs
    def paged_needs(self) -> List[Optional[PagedNeed]]:
        """Per run entry: the pages it owns (None if it owns none)."""
        out: List[Optional[PagedNeed]] = []
        for e in self.layout.order:
            out.append(None if e.reads_cache_of is not None else self.parts.mixers[e.layer].paged_need())
        return out

    def state_needs(self) -> Dict[int, StateNeed]:
        out: Dict[int, StateNeed] = {}
        for i, e in enumerate(self.layout.order):
            need = None if e.reads_cache_of is not None else self.parts.mixers[e.layer].state_need()
            if need is not None:
                out[i] = need
        return out

    def capturable(self) -> bool:
        """Whether every part's forward may be recorded into a HIP graph."""
        return all(getattr(p, "capturable", True) for p in self.parts.all_parts)

    def packed(self) -> bool:
        """Whether the matrices have their second copy in the streaming kernels' order."""
        return any(isinstance(v, StreamedMatrix) and v.packed is not None
                   for p in self.parts.all_parts for v in vars(p).values())

    def weight_bytes(self) -> int:
        seen, total = set(), 0
        for p in self.parts.all_parts:
            for v in vars(p).values():
                held = [v.rows, v.packed.data if v.packed is not None else None] if isinstance(v, StreamedMatrix) else [v]
                for t in held:
                    if isinstance(t, torch.Tensor) and t.data_ptr() not in seen:
                        seen.add(t.data_ptr())
                        total += t.numel() * t.element_size()
        return total

    # ------------------------------------------------------------- forward
    def forward(self, ctx: StepContext, stores: Sequence[LayerStore]) -> Optional[torch.Tensor]:
        """Run the step's tokens through every entry of the order; fp32
        logits ``[n_out, vocab]`` at ``ctx.out_rows`` (None when none is wanted;
        the cache is written all the same)."""
        if not self.loaded:
            raise RuntimeError("the model has no weights yet")
        h = self.parts.embed.forward(ctx.tokens, ctx)
        if self.layout.streams:
            h = streams_spread(h, self.layout.streams)  # [S, T, dim]: the blocks and the last norm know
        injections = self.parts.injections
        # the embedding's output as it was, for injections that add it again (h itself moves on)
        embedded = h.clone() if any(p.needs_embedding for p in injections) else None
        pending = None  # rows still to be added to h, or ScaledRows (added already, the next norm half done)
        blocks, order = self.parts.blocks, self.layout.order
        for i, entry in enumerate(order):
            block = blocks[entry.layer]
            if entry.inject is not None:
                if isinstance(pending, PostNormed):  # a sublayer's output that is normed before it is added
                    post_add_rmsnorm(h, pending.rows, pending.weight, pending.eps, None, 0.0, None, delta_bias=pending.bias)
                    pending = None
                if isinstance(pending, ScaledDelta):  # ... or that is scaled per channel
                    stream_add(h, pending.rows, None, None, delta_scale=pending.scale)
                    pending = None
                if isinstance(pending, StreamTerms) and not injections[entry.inject[0]].takes_terms:
                    stream_terms(h, pending)
                    pending = None
                injections[entry.inject[0]].forward(h, None if isinstance(pending, ScaledRows) else pending,
                                                    embedded, entry.inject[1])
                pending = None
            if getattr(block, "folds_norms", False):
                # the norm that follows this block is the next block's first, if that block can take over
                after = blocks[order[i + 1].layer] if i + 1 < len(order) and order[i + 1].inject is None else None
                next_norm = after.mixer_norm if getattr(after, "folds_norms", False) else None
                pending = block.forward(h, pending, ctx, stores[i], next_norm=next_norm)
            else:
                pending = block.forward(h, None if isinstance(pending, ScaledRows) else pending, ctx, stores[i])
        if isinstance(pending, ScaledRows):
            pending = None  # h holds the sum already
        if ctx.n_out == 0:
            return None
        x = self.parts.final_norm.forward(h, pending, ctx.act_dtype, rows=ctx.out_rows)
        return self.parts.head.forward(x)
