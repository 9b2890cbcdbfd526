"""The recurrent block of Griffin with a real-gated linear recurrent unit: a number per channel instead of keys.

``W_y x + b_y`` and ``W_x x + b_x`` (``width`` channels each); the second passes a short causal convolution per channel
(``taps`` taps and a bias), giving ``u``.  ``r`` and ``i`` are the sigmoids of two block-diagonal products of ``u`` (``blocks``
equal blocks, with biases); ``log a = -c r softplus(lam)``; the state moves as ``S <- a S + sqrt(1 - a^2) i u`` from zero;
the result ``S * gelu_tanh(y)`` is projected back.

The request's state slot holds, per channel, one fp32 row: ``S`` and behind it the convolution's last ``taps - 1``
inputs, so that a prompt may be cut anywhere.  Gates, decays, the state and the gelu are fp32 (``csrc/lru.hip``); the
convolution's output is rounded to the activation dtype, which is what the block-diagonal products take.

Options: ``dim``, ``width``, ``blocks``, ``taps``, ``decay_scale`` (c).
"""

from __future__ import annotations

from typing import Any, List, Mapping

import torch

from ..kernels import ops
from .base import VECTOR, LayerStore, StateNeed, TensorSpec, place, register_part, MATRIX
from .rows_mixer import RowsMixer


class GatedLinearRecurrence(RowsMixer):
    def __init__(self, spec) -> None:
        super().__init__(spec)
        o = spec.options
        self.dim = int(o["dim"])
        self.width = int(o["width"])
        self.blocks = int(o["blocks"])
        self.taps = int(o["taps"])
        self.decay_scale = float(o.get("decay_scale", 8.0))
        if min(self.width, self.blocks) <= 0 or self.width % self.blocks:
            raise ValueError(f"{self.prefix}: width={self.width} is not a multiple of blocks={self.blocks}")
        if not 1 <= self.taps <= ops.CONV_MAX_TAPS:
            raise ValueError(f"{self.prefix}: {self.taps} taps are not supported (1 to {ops.CONV_MAX_TAPS})")
        self.block = self.width // self.blocks
        self.in_width, self.out_width = 2 * self.width, self.width
        self.y_bias = self.x_bias = self.conv_w = self.conv_b = self.w_gates = self.gates_b = self.decay = None

    def tensor_specs(self) -> List[TensorSpec]:
        W, B, n = self.width, self.blocks, self.block
        return [TensorSpec(self._name("y_proj.weight"), (W, self.dim)), TensorSpec(self._name("y_proj.bias"), (W,), VECTOR, ("normal", 0.1)),
                TensorSpec(self._name("x_proj.weight"), (W, self.dim)), TensorSpec(self._name("x_proj.bias"), (W,), VECTOR, ("normal", 0.1)),
                TensorSpec(self._name("conv.weight"), (W, self.taps), VECTOR, ("normal", 0.3)),
                TensorSpec(self._name("conv.bias"), (W,), VECTOR, ("normal", 0.1)),
                TensorSpec(self._name("r_gate.weight"), (B, n, n), MATRIX, ("normal", 0.05)),
                TensorSpec(self._name("r_gate.bias"), (B, n), VECTOR, ("normal", 0.5)),
                TensorSpec(self._name("i_gate.weight"), (B, n, n), MATRIX, ("normal", 0.05)),
                TensorSpec(self._name("i_gate.bias"), (B, n), VECTOR, ("normal", 0.5)),
                TensorSpec(self._name("decay"), (W,), VECTOR, ("normal", 1.0)),
                TensorSpec(self._name("o_proj.weight"), (self.dim, W))]

    def in_matrix(self, tensors: Mapping[str, torch.Tensor]) -> torch.Tensor:
        return torch.cat([tensors[self._name("y_proj.weight")], tensors[self._name("x_proj.weight")]])

    def out_matrix(self, tensors: Mapping[str, torch.Tensor]) -> torch.Tensor:
        return tensors[self._name("o_proj.weight")]

    def load_rest(self, tensors: Mapping[str, torch.Tensor], dtype: torch.dtype, device: Any) -> None:
        t = lambda name: tensors[self._name(name)]
        f32 = lambda name: t(name).to(device=device, dtype=torch.float32).contiguous()
        self.y_bias, self.x_bias, self.conv_w, self.conv_b = f32("y_proj.bias"), f32("x_proj.bias"), f32("conv.weight"), f32("conv.bias")
        # per block: the rows of r, then the rows of i
        self.w_gates = place(torch.cat([t("r_gate.weight"), t("i_gate.weight")], dim=1), MATRIX, dtype, device)
        self.gates_b = torch.cat([f32("r_gate.bias"), f32("i_gate.bias")], dim=1).contiguous()
        self.decay = (self.decay_scale * torch.nn.functional.softplus(f32("decay"))).contiguous()

    def state_need(self) -> StateNeed:
        return StateNeed((self.width, self.taps), torch.float32)

    def mix(self, rows: torch.Tensor, ctx: Any, store: LayerStore, out: torch.Tensor, out_scale: float = 1.0) -> None:
        W, T = self.width, rows.shape[0]
        x = rows[:, W:]
        u = torch.empty((T, -(-W // 8) * 8), dtype=out.dtype, device=out.device)
        ops.causal_conv(x, self.conv_w, self.conv_b, store.state, 1, ctx.slot_ids, ctx.seq_of_token, ctx.q_start, u,
                        in_bias=self.x_bias)
        gates = torch.empty((T, 2 * W), dtype=torch.float32, device=out.device)
        ops.head_linear(u, self.block, self.w_gates, gates, 2 * self.block, bias=self.gates_b)
        ops.lru_scan(u, gates, self.block, self.decay, rows, self.y_bias, out_scale, x, self.x_bias, self.taps, store.state,
                     ctx.slot_ids, ctx.q_start, ctx.n_seqs, out, q_start_host=None if ctx.graph_capacity else ctx.q_start_host)


register_part("mixer", "gated_linear_recurrence", GatedLinearRecurrence)
