"""Mixers of the form ``W_out m(W_in x)``, and two of them side by side on the same input.

A :class:`RowsMixer` says which matrix makes its rows from the layer's input, which matrix takes its result back, and
what happens between (:meth:`RowsMixer.mix`).  Alone it is a mixer like the others; :class:`ParallelMixers` runs two of
them on one input as one product in (both matrices stacked) and one product out (their results side by side, the two
constant factors applied where each result is rounded): ``left_scale * left(x) + right_scale * right(x)``.

With ``out_norms`` the two results have an output product each, and the mixer's output is ``left_scale * n(left(x)) (.) w_l +
right_scale * n(right(x)) (.) w_r`` with ``n`` the division by the root mean square over the model's width (``eps``): it is
returned as terms (:class:`~fastgen_amd.kernels.ops.StreamTerms`), which the kernel that adds them to the stream norms.

``ParallelMixers`` options: ``dim``, ``left``, ``right`` (:class:`~fastgen_amd.config.PartSpec` of mixers of this form, with
tensor names of their own), ``left_scale``, ``right_scale``, ``out_norms``, ``eps``.  At most one of the two keeps pages, at most one a state.
"""

from __future__ import annotations

from typing import Any, List, Mapping, Optional

import torch

from ..kernels import ops
from ..kernels.linear import StreamedMatrix, linear, streamed
from .base import MATRIX, VECTOR, LayerStore, Mixer, PagedNeed, StateNeed, TensorSpec, build_part, place, register_part


def _padded(n: int) -> int:
    return -(-n // 8) * 8  # what the products' kernels read and write at once


def load_in(w: torch.Tensor, dtype: torch.dtype, device: Any) -> StreamedMatrix:
    """An input matrix with zero rows up to a multiple of 8."""
    pad = _padded(w.shape[0]) - w.shape[0]
    return streamed(place(torch.cat([w, w.new_zeros(pad, w.shape[1])]) if pad else w, MATRIX, dtype, device))


def load_out(w: torch.Tensor, dtype: torch.dtype, device: Any) -> StreamedMatrix:
    """An output matrix with zero columns up to a multiple of 8."""
    pad = _padded(w.shape[1]) - w.shape[1]
    return streamed(place(torch.cat([w, w.new_zeros(w.shape[0], pad)], dim=1) if pad else w, MATRIX, dtype, device))


def result_rows(T: int, width: int, dtype: torch.dtype, device: Any) -> torch.Tensor:
    """Room for results of ``width`` columns, padded (with zeros) to what :func:`load_out` made of the matrix."""
    wide = _padded(width)
    return (torch.empty if wide == width else torch.zeros)((T, wide), dtype=dtype, device=device)


class RowsMixer(Mixer):
    """``in_matrix`` / ``out_matrix`` give the two matrices from the checkpoint's tensors, ``load_rest`` takes the other
    tensors, ``mix`` writes the result's ``out_width`` columns (times ``out_scale``, rounded once) from the fp32 rows of the
    input product, of which this mixer's columns begin at ``rows``' first."""

    in_width: int
    out_width: int

    def in_matrix(self, tensors: Mapping[str, torch.Tensor]) -> torch.Tensor:
        raise NotImplementedError

    def out_matrix(self, tensors: Mapping[str, torch.Tensor]) -> torch.Tensor:
        raise NotImplementedError

    def load_rest(self, tensors: Mapping[str, torch.Tensor], dtype: torch.dtype, device: Any) -> None:
        raise NotImplementedError

    def mix(self, rows: torch.Tensor, ctx: Any, store: LayerStore, out: torch.Tensor, out_scale: float = 1.0) -> None:
        raise NotImplementedError

    w_in: Optional[StreamedMatrix] = None
    wo: Optional[StreamedMatrix] = None

    def load(self, tensors: Mapping[str, torch.Tensor], dtype: torch.dtype, device: Any) -> None:
        self.w_in = load_in(self.in_matrix(tensors), dtype, device)
        self.wo = load_out(self.out_matrix(tensors), dtype, device)
        self.load_rest(tensors, dtype, device)

    def forward(self, x: torch.Tensor, ctx: Any, store: LayerStore) -> torch.Tensor:
        rows = linear(x, self.w_in, out_dtype=torch.float32)
        out = result_rows(x.shape[0], self.out_width, x.dtype, x.device)
        self.mix(rows, ctx, store, out)
        return linear(out, self.wo, partials_ok=True)


class ParallelMixers(Mixer):
    def __init__(self, spec) -> None:
        super().__init__(spec)
        o = spec.options
        self.dim = int(o["dim"])
        self.left: RowsMixer = build_part("mixer", o["left"])
        self.right: RowsMixer = build_part("mixer", o["right"])
        self.scales = (float(o.get("left_scale", 1.0)), float(o.get("right_scale", 1.0)))
        for side in (self.left, self.right):
            if not isinstance(side, RowsMixer):
                raise ValueError(f"{self.prefix}: {side.spec.kind!r} is no mixer that can run beside another on one product")
        if all(s.paged_need() is not None for s in self.sides) or all(s.state_need() is not None for s in self.sides):
            raise ValueError(f"{self.prefix}: of two mixers side by side at most one keeps pages and at most one a state")
        self.capturable = all(s.capturable for s in self.sides)
        self.w_in: Optional[StreamedMatrix] = None
        self.wo: Optional[StreamedMatrix] = None
        self.returns_terms = bool(o.get("out_norms", False))
        self.eps = float(o.get("eps", 0.0))
        self.right_col = _padded(self.left.in_width)  # (the right side's columns begin where its kernels can read them as vectors)
        self.wo_right: Optional[StreamedMatrix] = None
        self.out_scales: List[torch.Tensor] = []

    @property
    def sides(self):
        return (self.left, self.right)

    def tensor_specs(self) -> List[TensorSpec]:
        norms = [TensorSpec(self._name(f"{n}_norm.weight"), (self.dim,), VECTOR, ("one_plus_normal", 0.1)) for n in ("left", "right")]
        return self.left.tensor_specs() + self.right.tensor_specs() + (norms if self.returns_terms else [])

    def load(self, tensors: Mapping[str, torch.Tensor], dtype: torch.dtype, device: Any) -> None:
        mats = [s.in_matrix(tensors) for s in self.sides]
        gap = mats[0].new_zeros(self.right_col - self.left.in_width, self.dim)
        self.w_in = load_in(torch.cat([mats[0], gap, mats[1]]), dtype, device)
        for s in self.sides:
            s.load_rest(tensors, dtype, device)
        if not self.returns_terms:
            self.wo = load_out(torch.cat([s.out_matrix(tensors) for s in self.sides], dim=1), dtype, device)
            return
        self.wo, self.wo_right = (load_out(s.out_matrix(tensors), dtype, device) for s in self.sides)
        self.out_scales = [(c * tensors[self._name(f"{n}_norm.weight")].to(device=device, dtype=torch.float32)).contiguous()
                           for n, c in zip(("left", "right"), self.scales)]

    def fold_scale(self, scale: torch.Tensor) -> None:
        """A vector that multiplies this mixer's terms is folded into their own (once, behind ``load``)."""
        self.out_scales = [(s * scale).contiguous() for s in self.out_scales]

    def paged_need(self) -> Optional[PagedNeed]:
        return self.left.paged_need() or self.right.paged_need()

    def state_need(self) -> Optional[StateNeed]:
        return self.left.state_need() or self.right.state_need()

    def forward(self, x: torch.Tensor, ctx: Any, store: LayerStore) -> torch.Tensor:
        rows = linear(x, self.w_in, out_dtype=torch.float32)
        if self.returns_terms:
            terms = []
            for s, own, w, scale in ((self.left, rows[:, : self.left.in_width], self.wo, self.out_scales[0]),
                                     (self.right, rows[:, self.right_col :], self.wo_right, self.out_scales[1])):
                out = result_rows(x.shape[0], s.out_width, x.dtype, x.device)
                s.mix(own, ctx, store, out)
                terms.append(ops.StreamTerm(linear(out, w, partials_ok=True), scale, None, self.eps))
            return ops.StreamTerms(terms)
        out = result_rows(x.shape[0], self.left.out_width + self.right.out_width, x.dtype, x.device)
        self.left.mix(rows[:, : self.left.in_width], ctx, store, out, self.scales[0])
        self.right.mix(rows[:, self.right_col :], ctx, store, out[:, self.left.out_width :], self.scales[1])
        return linear(out, self.wo, partials_ok=True)


register_part("mixer", "parallel_mixers", ParallelMixers)
