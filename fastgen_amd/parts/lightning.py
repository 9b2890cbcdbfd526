"""Linear attention whose state fades by a constant per head, and nothing else: a matrix per head instead of keys.

``q = silu(W_q x)``, ``k = silu(W_k x)`` (``n_heads`` heads of ``head_dim``), ``v = silu(W_v x)`` (of ``v_head_dim``); per head
``S <- decay_h S + k v^T``, ``o = S^T q`` from zero.  The heads' outputs are normed together (one RMS norm over all
columns), multiplied by ``sigmoid(W_g x)`` and projected.  The state lives in fp32 in the request's slot
(``csrc/lightning.hip``: token by token for decoded tokens and short portions, in chunks side by side for prompts).

Options: ``dim``, ``n_heads``, ``head_dim``, ``v_head_dim``, ``decay`` (a number per head, in 0 .. 1), ``eps``.
"""

from __future__ import annotations

import math
from typing import Any, List, Mapping

import torch

from ..kernels import ops
from .base import VECTOR, LayerStore, StateNeed, TensorSpec, register_part
from .rows_mixer import RowsMixer


class LightningAttention(RowsMixer):
    def __init__(self, spec) -> None:
        super().__init__(spec)
        o = spec.options
        self.dim = int(o["dim"])
        self.n_heads = int(o["n_heads"])
        self.head_dim = int(o["head_dim"])
        self.v_head_dim = int(o["v_head_dim"])
        self.eps = float(o["eps"])
        self.decay = [float(x) for x in o["decay"]]
        if len(self.decay) != self.n_heads or not all(0 <= x <= 1 for x in self.decay):
            raise ValueError(f"{self.prefix}: {self.n_heads} heads need as many decays between 0 and 1")
        if not 0 < self.head_dim <= 512 or self.v_head_dim < 1:
            raise ValueError(f"{self.prefix}: heads of {self.head_dim} x {self.v_head_dim} are not supported (at most 512 key channels)")
        H, d, e = self.n_heads, self.head_dim, self.v_head_dim
        if H * e > 16384:
            raise ValueError(f"{self.prefix}: {H * e} value columns are not supported (at most 16384)")
        self.in_width, self.out_width = 2 * H * d + 2 * H * e, H * e
        self.log_decay = self.norm_w = None

    def tensor_specs(self) -> List[TensorSpec]:
        H, d, e = self.n_heads, self.head_dim, self.v_head_dim
        return [TensorSpec(self._name(f"{n}_proj.weight"), (H * c, self.dim)) for n, c in (("q", d), ("k", d), ("v", e), ("gate", e))] + [
            TensorSpec(self._name("out_norm.weight"), (H * e,), VECTOR, ("one_plus_normal", 0.01)),
            TensorSpec(self._name("o_proj.weight"), (self.dim, H * e))]

    def in_matrix(self, tensors: Mapping[str, torch.Tensor]) -> torch.Tensor:
        return torch.cat([tensors[self._name(f"{n}_proj.weight")] for n in ("q", "k", "v", "gate")])

    def out_matrix(self, tensors: Mapping[str, torch.Tensor]) -> torch.Tensor:
        return tensors[self._name("o_proj.weight")]

    def load_rest(self, tensors: Mapping[str, torch.Tensor], dtype: torch.dtype, device: Any) -> None:
        # (a decay of zero: a logarithm whose multiples are still numbers, and whose exponentials are zero)
        logs = [math.log(x) if x > 0 else -1e4 for x in self.decay]
        self.log_decay = torch.tensor(logs, dtype=torch.float32, device=device)
        self.norm_w = tensors[self._name("out_norm.weight")].to(device=device, dtype=torch.float32).contiguous()

    def state_need(self) -> StateNeed:
        return StateNeed((self.n_heads, self.head_dim, self.v_head_dim), torch.float32)

    def mix(self, rows: torch.Tensor, ctx: Any, store: LayerStore, out: torch.Tensor, out_scale: float = 1.0) -> None:
        H, d, e = self.n_heads, self.head_dim, self.v_head_dim
        o = torch.empty((rows.shape[0], H * e), dtype=torch.float32, device=rows.device)
        ops.lightning_scan(rows, 0, H * d, 2 * H * d, self.log_decay, store.state, ctx.slot_ids, ctx.q_start, ctx.n_seqs, o,
                           q_start_host=None if ctx.graph_capacity else ctx.q_start_host)
        ops.row_norm_gate(o, self.norm_w, self.eps, rows[:, 2 * H * d + H * e :], out, out_scale)


register_part("mixer", "lightning_attention", LightningAttention)
