"""The gated delta rule: a recurrence on a matrix per head instead of a cache of keys.

q and k (``n_kv_heads`` heads of ``head_dim``) and v (``n_heads`` heads of ``v_head_dim``) each pass a short causal convolution
per channel and SiLU; q and k become unit vectors per head, q times ``head_dim^-1/2``.  Per value head (query/key head
``h // (n_heads / n_kv_heads)``) a state ``S [head_dim, v_head_dim]`` moves as

    S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q

with ``beta = sigmoid(W_b x)`` and ``g = exp(-exp(A_log) softplus(W_a x + dt_bias))`` per head.  Each head's output is divided
by its root mean square, multiplied by one weight for all heads and by ``silu(W_g x)``, and projected.

The request's state slot holds the heads' states in fp32 and behind them the convolutions' last ``taps - 1`` inputs,
channel by channel.  Everything from the product's fp32 rows to the gate is fp32 (``csrc/delta_rule.hip``).

``channel_delta_rule`` is the same with a decay per head and key channel, ``S <- diag(g) S`` with ``g = exp(-exp(A_log)
softplus(W_a2 (W_a1 x) + dt_bias))`` (``[n_heads, head_dim]``, through a narrow middle of ``decay_rank``), and an output gate
``sigmoid(W_g2 (W_g1 x))`` through a narrow middle of ``gate_rank``.  Both second halves are one launch
(``csrc/low_rank.hip``), which leaves the decays' logarithms where the recurrence reads them.

Options: ``dim``, ``n_heads``, ``n_kv_heads``, ``head_dim``, ``v_head_dim``, ``taps``, ``eps``, ``unit_eps`` (inside the root
of the unit vectors' norm).
"""

from __future__ import annotations

from typing import Any, List, Mapping

import torch

from ..kernels import ops
from .base import MATRIX, VECTOR, LayerStore, StateNeed, TensorSpec, place, register_part
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

    def _conv_specs(self) -> List[TensorSpec]:
        """The projections of q, k and v and their convolutions."""
        G, d, e = self.n_kv_heads, self.head_dim, self.v_head_dim
        specs = []
        for n, c in (("q", G * d), ("k", G * d), ("v", self.n_heads * e)):
            specs += [TensorSpec(self._name(f"{n}_proj.weight"), (c, self.dim)),
                      TensorSpec(self._name(f"{n}_conv.weight"), (c, self.taps), VECTOR, ("normal", 0.5))]
        return specs

    def tensor_specs(self) -> List[TensorSpec]:
        H, e = self.n_heads, self.v_head_dim
        return self._conv_specs() + [
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

    def _state(self, ctx: Any, store: LayerStore):
        """The heads' states ``[n_slots, H, d, e]`` and the convolutions' operands, from the request's slots."""
        slots = store.state.shape[0]
        S = store.state[:, : self._matrix].view(slots, self.n_heads, self.head_dim, self.v_head_dim)
        tails = store.state[:, self._matrix :].view(slots, self.channels, -1)
        moves = ctx.graph_capacity > 0 or ctx.max_q_len == 1
        return S, ops.ConvInputs(self.conv_w, tails, 0, ctx.slot_ids, ctx.seq_of_token, ctx.q_start, moves)

    def mix(self, rows: torch.Tensor, ctx: Any, store: LayerStore, out: torch.Tensor, out_scale: float = 1.0) -> None:
        H, G, d, e, C = self.n_heads, self.n_kv_heads, self.head_dim, self.v_head_dim, self.channels
        T = rows.shape[0]
        S, conv = self._state(ctx, store)
        # (rows of a multiple of 4: the chunked scan reads them as vectors)
        ready = torch.empty((T, -(-(C + 2 * H) // 4) * 4), dtype=torch.float32, device=rows.device)
        ops.delta_prepare(rows, G, d, H, e, conv, C + H * e, C + H * e + H, self.decay_rate, self.dt_bias, d ** -0.5,
                          self.unit_eps, ready)
        if not conv.moves:
            ops.conv_tail(rows, conv, ctx.n_seqs)
        o = torch.empty((T, H * e), dtype=torch.float32, device=rows.device)
        ops.delta_scan(ready, G, d, H, e, S, ctx.slot_ids, ctx.q_start, ctx.n_seqs, o,
                       q_start_host=None if ctx.graph_capacity else ctx.q_start_host)
        ops.head_norm_gate(o, self.norm_w, self.eps, rows[:, C:], H, out[:, : H * e], out_scale)


class ChannelDeltaRule(GatedDeltaRule):
    def __init__(self, spec) -> None:
        super().__init__(spec)
        o = spec.options
        self.decay_rank, self.gate_rank = int(o["decay_rank"]), int(o["gate_rank"])
        if min(self.decay_rank, self.gate_rank) < 1:
            raise ValueError(f"{self.prefix}: the narrow middles must be at least one wide")
        up8 = lambda n: -(-n // 8) * 8
        # columns of the product: q, k, v, the two narrow middles (each on a multiple of 8, what the second halves'
        # kernel reads at once), beta
        self.a_col = up8(self.channels)
        self.g_col = self.a_col + up8(self.decay_rank)
        self.b_col = self.g_col + up8(self.gate_rank)
        self.in_width = self.b_col + self.n_heads
        self.w_a2 = self.w_g2 = None

    def tensor_specs(self) -> List[TensorSpec]:
        H, d, e = self.n_heads, self.head_dim, self.v_head_dim
        return self._conv_specs() + [
            TensorSpec(self._name("beta_proj.weight"), (H, self.dim)), TensorSpec(self._name("A_log"), (H,), VECTOR, ("normal", 0.5)),
            TensorSpec(self._name("decay_down.weight"), (self.decay_rank, self.dim)),
            TensorSpec(self._name("decay_up.weight"), (H * d, self.decay_rank)),
            TensorSpec(self._name("dt_bias"), (H * d,), VECTOR, ("normal", 1.0)),
            TensorSpec(self._name("gate_down.weight"), (self.gate_rank, self.dim)),
            TensorSpec(self._name("gate_up.weight"), (H * e, self.gate_rank)),
            TensorSpec(self._name("out_norm.weight"), (e,), VECTOR, ("one_plus_normal", 0.01)),
            TensorSpec(self._name("o_proj.weight"), (self.dim, H * e))]

    def in_matrix(self, tensors: Mapping[str, torch.Tensor]) -> torch.Tensor:
        t = lambda name: tensors[self._name(name)]
        out = t("q_proj.weight").new_zeros(self.in_width, self.dim)
        at = 0
        for n in ("q", "k", "v"):
            w = t(f"{n}_proj.weight")
            out[at : at + w.shape[0]] = w
            at += w.shape[0]
        for col, n in ((self.a_col, "decay_down"), (self.g_col, "gate_down"), (self.b_col, "beta_proj")):
            w = t(f"{n}.weight")
            out[col : col + w.shape[0]] = w
        return out

    def load_rest(self, tensors: Mapping[str, torch.Tensor], dtype: torch.dtype, device: Any) -> None:
        super().load_rest(tensors, dtype, device)

        def second(name: str) -> torch.Tensor:  # zero columns meet the padding of the middle
            w = tensors[self._name(name)]
            return place(torch.cat([w, w.new_zeros(w.shape[0], -w.shape[1] % 8)], dim=1), MATRIX, dtype, device)

        self.w_a2, self.w_g2 = second("decay_up.weight"), second("gate_up.weight")

    def mix(self, rows: torch.Tensor, ctx: Any, store: LayerStore, out: torch.Tensor, out_scale: float = 1.0) -> None:
        H, G, d, e, C = self.n_heads, self.n_kv_heads, self.head_dim, self.v_head_dim, self.channels
        T = rows.shape[0]
        S, conv = self._state(ctx, store)
        # what the recurrence takes of a token: [q | k | v | beta | log g per channel], runs on multiples of 4
        log_col = -(-(C + H) // 4) * 4
        ready = torch.empty((T, -(-(log_col + H * d) // 4) * 4), dtype=torch.float32, device=rows.device)
        gate = torch.empty((T, H * e), dtype=torch.float32, device=rows.device)
        ops.delta_prepare(rows, G, d, H, e, conv, self.b_col, -1, None, None, d ** -0.5, self.unit_eps, ready)
        if not conv.moves:
            ops.conv_tail(rows, conv, ctx.n_seqs)
        ops.low_rank(rows, [ops.LowRankJob(self.a_col, self.w_a2, ready[:, log_col:], self.dt_bias, self.decay_rate, d),
                            ops.LowRankJob(self.g_col, self.w_g2, gate)])
        o = torch.empty((T, H * e), dtype=torch.float32, device=rows.device)
        ops.delta_scan(ready, G, d, H, e, S, ctx.slot_ids, ctx.q_start, ctx.n_seqs, o,
                       q_start_host=None if ctx.graph_capacity else ctx.q_start_host, channel_decay_col=log_col)
        ops.head_norm_gate(o, self.norm_w, self.eps, gate, H, out[:, : H * e], out_scale, sigmoid=True)


register_part("mixer", "gated_delta_rule", GatedDeltaRule)
register_part("mixer", "channel_delta_rule", ChannelDeltaRule)
