"""The gated delta rule: a recurrence on a matrix per head instead of a cache of keys.

q and k (``n_kv_heads`` heads of ``head_dim``) and v (``n_heads`` heads of ``v_head_dim``) each pass a short causal convolution
per channel and SiLU; q and k become unit vectors per head, q times ``head_dim^-1/2``.  Per value head (query/key head
``h // (n_heads / n_kv_heads)``) a state ``S [head_dim, v_head_dim]`` moves as

    S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q

with ``beta = sigmoid(W_b x)`` and ``g = exp(-exp(A_log) softplus(W_a x + dt_bias))`` per head.  Each head's output is divided
by its root mean square, multiplied by one weight for all heads and by ``silu(W_g x)``, and projected.

The request's state slot holds the heads' states in fp32 and behind them the convolutions' last ``taps - 1`` inputs,
channel by channel.  Everything from the product's fp32 rows to the gate is fp32 (``csrc/delta_rule.hip``).

Options: ``dim``, ``n_heads``, ``n_kv_heads``, ``head_dim``, ``v_head_dim``, ``taps``, ``eps``, ``unit_eps`` (inside the root
of the unit vectors' norm).
"""

from __future__ import annotations

from typing import Any, List, Mapping

import torch

from ..kernels import ops
from .base import VECTOR, LayerStore, StateNeed, TensorSpec, register_part
from .rows_mixer import RowsMixer


class GatedDeltaRule(RowsMixer):
    def __init__(self, spec) -> None:
        super().__init__(spec)
        o = spec.options
        self.dim = int(o["dim"])
        self.n_heads = int(o["n_heads"])
        self.n_kv_heads = int(o["n_kv_heads"])
        self.head_dim = int(o["head_dim"])
        self.v_head_dim = int(o["v_head_dim"])
        self.taps = int(o["taps"])
        self.eps = float(o["eps"])
        self.unit_eps = float(o.get("unit_eps", 1e-6))
        if self.n_heads % self.n_kv_heads:
            raise ValueError(f"{self.prefix}: n_heads={self.n_heads} is not a multiple of n_kv_heads={self.n_kv_heads}")
        if self.head_dim <= 0 or self.v_head_dim <= 0 or self.head_dim % 2 or self.v_head_dim % 2 or self.head_dim > 512 \
                or self.v_head_dim > 1024:
            raise ValueError(f"{self.prefix}: heads of {self.head_dim} x {self.v_head_dim} are not supported"
                             " (even, at most 512 key channels and 1024 value channels)")
        if not 1 <= self.taps <= ops.CONV_MAX_TAPS:
            raise ValueError(f"{self.prefix}: {self.taps} taps are not supported (1 to {ops.CONV_MAX_TAPS})")
        H, G, d, e = self.n_heads, self.n_kv_heads, self.head_dim, self.v_head_dim
        self.channels = 2 * G * d + H * e  # q, k, v: what the convolutions run over
        self.in_width, self.out_width = self.channels + H * e + 2 * H, H * e
        self.conv_w = self.decay_rate = self.dt_bias = self.norm_w = None

    def tensor_specs(self) -> List[TensorSpec]:
        H, G, d, e = self.n_heads, self.n_kv_heads, self.head_dim, self.v_head_dim
        specs = []
        for n, c in (("q", G * d), ("k", G * d), ("v", H * e)):
            specs += [TensorSpec(self._name(f"{n}_proj.weight"), (c, self.dim)),
                      TensorSpec(self._name(f"{n}_conv.weight"), (c, self.taps), VECTOR, ("normal", 0.5))]
        return specs + [
            TensorSpec(self._name("gate_proj.weight"), (H * e, self.dim)),
            TensorSpec(self._name("beta_proj.weight"), (H, self.dim)), TensorSpec(self._name("decay_proj.weight"), (H, self.dim)),
            TensorSpec(self._name("A_log"), (H,), VECTOR, ("normal", 0.5)), TensorSpec(self._name("dt_bias"), (H,), VECTOR, ("normal", 1.0)),
            TensorSpec(self._name("out_norm.weight"), (e,), VECTOR, ("one_plus_normal", 0.01)),
            TensorSpec(self._name("o_proj.weight"), (self.dim, H * e))]

    def in_matrix(self, tensors: Mapping[str, torch.Tensor]) -> torch.Tensor:
        return torch.cat([tensors[self._name(f"{n}_proj.weight")] for n in ("q", "k", "v", "gate", "beta", "decay")])

    def out_matrix(self, tensors: Mapping[str, torch.Tensor]) -> torch.Tensor:
        return tensors[self._name("o_proj.weight")]

    def load_rest(self, tensors: Mapping[str, torch.Tensor], dtype: torch.dtype, device: Any) -> None:
        f32 = lambda name: tensors[self._name(name)].to(device=device, dtype=torch.float32).contiguous()
        self.conv_w = torch.cat([f32(f"{n}_conv.weight") for n in ("q", "k", "v")]).contiguous()
        self.decay_rate, self.dt_bias, self.norm_w = torch.exp(f32("A_log")).contiguous(), f32("dt_bias"), f32("out_norm.weight")

    @property
    def _matrix(self) -> int:
        return self.n_heads * self.head_dim * self.v_head_dim

    def state_need(self) -> StateNeed:
        # the heads' matrices, then the convolutions' tails (one column where there is one tap: never empty)
        return StateNeed((self._matrix + self.channels * max(1, self.taps - 1),), torch.float32)

    def mix(self, rows: torch.Tensor, ctx: Any, store: LayerStore, out: torch.Tensor, out_scale: float = 1.0) -> None:
        H, G, d, e, C = self.n_heads, self.n_kv_heads, self.head_dim, self.v_head_dim, self.channels
        T, slots = rows.shape[0], store.state.shape[0]
        S = store.state[:, : self._matrix].view(slots, H, d, e)
        tails = store.state[:, self._matrix :].view(slots, C, -1)
        moves = ctx.graph_capacity > 0 or ctx.max_q_len == 1
        conv = ops.ConvInputs(self.conv_w, tails, 0, ctx.slot_ids, ctx.seq_of_token, ctx.q_start, moves)
        # (rows of a multiple of 4: the chunked scan reads them as vectors)
        ready = torch.empty((T, -(-(C + 2 * H) // 4) * 4), dtype=torch.float32, device=rows.device)
        ops.delta_prepare(rows, G, d, H, e, conv, C + H * e, C + H * e + H, self.decay_rate, self.dt_bias, d ** -0.5,
                          self.unit_eps, ready)
        if not moves:
            ops.conv_tail(rows, conv, ctx.n_seqs)
        o = torch.empty((T, H * e), dtype=torch.float32, device=rows.device)
        ops.delta_scan(ready, G, d, H, e, S, ctx.slot_ids, ctx.q_start, ctx.n_seqs, o,
                       q_start_host=None if ctx.graph_capacity else ctx.q_start_host)
        ops.head_norm_gate(o, self.norm_w, self.eps, rows[:, C:], H, out[:, : H * e], out_scale)


register_part("mixer", "gated_delta_rule", GatedDeltaRule)
