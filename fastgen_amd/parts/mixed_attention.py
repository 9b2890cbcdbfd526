"""Grouped-query causal softmax attention whose heads' weights are mixed after the softmax.

Per step: one product for q, k and v (fp32 rows); an RMS norm over all of a token's query columns and one over all its
key columns (weights per column), rotation, keys and values into the pages, in one kernel; then attention: scores
through ``softcap * tanh(score / softcap)``, a sliding window, an ordinary softmax, and for every (query, key) pair the
heads' weights mixed by a matrix ``talk [H, H]`` before they meet the values (head ``h`` applies its mixed weights to the
values of its own key/value head); output projection.  Scores, weights and mixing are fp32.

Options: ``dim``, ``n_heads``, ``n_kv_heads``, ``head_dim``, ``v_head_dim``, ``scale``, ``softcap`` (None: none), ``window``,
``eps`` (of the two norms), ``position`` (a rotary scheme or none).
"""

from __future__ import annotations

from typing import Any, List, Mapping, Optional

import numpy as np
import torch

from ..kernels import ops
from .base import VECTOR, LayerStore, PagedNeed, TensorSpec, build_part, register_part
from .rows_mixer import RowsMixer


class MixedAttention(RowsMixer):
    def __init__(self, spec) -> None:
        super().__init__(spec)
        o = spec.options
        self.dim = int(o["dim"])
        self.n_heads = int(o["n_heads"])
        self.n_kv_heads = int(o["n_kv_heads"])
        self.head_dim = int(o["head_dim"])
        self.v_head_dim = int(o.get("v_head_dim") or self.head_dim)
        self.scale = float(o.get("scale", self.head_dim ** -0.5))
        self.softcap = float(o.get("softcap") or 0.0)
        self.window: Optional[int] = o.get("window") or None
        self.eps = float(o["eps"])
        if self.n_heads % self.n_kv_heads:
            raise ValueError(f"{self.prefix}: n_heads={self.n_heads} is not a multiple of n_kv_heads={self.n_kv_heads}")
        for name, v in (("head_dim", self.head_dim), ("v_head_dim", self.v_head_dim)):
            if v <= 0 or v % 2:
                raise ValueError(f"{self.prefix}: {name}={v} must be positive and even")
        # a head in the cache: keys and values padded with zeros to one width, a multiple of 16
        self.cache_dim = -(-max(self.head_dim, self.v_head_dim) // 16) * 16
        if self.cache_dim > 512:
            raise ValueError(f"{self.prefix}: heads of {max(self.head_dim, self.v_head_dim)} are more than the attention kernels' 512")
        self.position = build_part("position", o["position"])
        self.in_width = self.n_heads * self.head_dim + self.n_kv_heads * (self.head_dim + self.v_head_dim)
        self.out_width = self.n_heads * self.v_head_dim
        self.freqs = self.q_norm_w = self.k_norm_w = self.talk = None
        self.talk_low = True

    def tensor_specs(self) -> List[TensorSpec]:
        H, G, d, e = self.n_heads, self.n_kv_heads, self.head_dim, self.v_head_dim
        return [TensorSpec(self._name("q_proj.weight"), (H * d, self.dim)), TensorSpec(self._name("k_proj.weight"), (G * d, self.dim)),
                TensorSpec(self._name("v_proj.weight"), (G * e, self.dim)),
                TensorSpec(self._name("q_norm.weight"), (H * d,), VECTOR, ("one_plus_normal", 0.1)),
                TensorSpec(self._name("k_norm.weight"), (G * d,), VECTOR, ("one_plus_normal", 0.1)),
                TensorSpec(self._name("head_mix"), (H, H), VECTOR, ("eye_plus_normal", 0.2)),
                TensorSpec(self._name("o_proj.weight"), (self.dim, H * e))]

    def in_matrix(self, tensors: Mapping[str, torch.Tensor]) -> torch.Tensor:
        t = lambda name: tensors[self._name(name)]
        return torch.cat([self.position.arrange_rows(t("q_proj.weight"), self.n_heads),
                          self.position.arrange_rows(t("k_proj.weight"), self.n_kv_heads), t("v_proj.weight")])

    def out_matrix(self, tensors: Mapping[str, torch.Tensor]) -> torch.Tensor:
        return tensors[self._name("o_proj.weight")]

    def load_rest(self, tensors: Mapping[str, torch.Tensor], dtype: torch.dtype, device: Any) -> None:
        f32 = lambda t: t.to(device=device, dtype=torch.float32).contiguous()
        # the norms' weights move with the rows that the rotation's pairing rearranges
        arranged = lambda name, n: self.position.arrange_rows(tensors[self._name(name)][:, None], n)[:, 0]
        self.q_norm_w = f32(arranged("q_norm.weight", self.n_heads))
        self.k_norm_w = f32(arranged("k_norm.weight", self.n_kv_heads))
        self.talk = f32(tensors[self._name("head_mix")])
        self.talk_low = not bool(torch.equal(self.talk, self.talk.to(torch.bfloat16).float()))
        self.freqs = self.position.frequencies_on(device)

    def paged_need(self) -> PagedNeed:
        return PagedNeed(self.n_kv_heads, self.cache_dim, self.window)

    def _rope_table(self, ctx: Any):
        if self.freqs is None:
            return None
        key = ("rope_table", self.freqs.data_ptr())
        table = ctx.scratch.get(key)
        if table is None:
            table = ctx.scratch[key] = ops.rope_table(ctx.positions, self.freqs)
        return table

    def mix(self, rows: torch.Tensor, ctx: Any, store: LayerStore, out: torch.Tensor, out_scale: float = 1.0) -> None:
        H, G, d, e = self.n_heads, self.n_kv_heads, self.head_dim, self.v_head_dim
        group = ctx.groups[store.group]
        q = torch.empty((rows.shape[0], H * d), dtype=out.dtype, device=out.device)
        ops.heads_prepare(
            rows, None, self.eps, n_q=H, q_col=0, q_width=d, q_norm=self.q_norm_w, q_norm_dims=d, q_out=q, q_out_width=d,
            n_kv=G, k_col=H * d, k_width=d, k_norm=self.k_norm_w, k_norm_dims=d, v_col=(H + G) * d, v_width=e,
            table=self._rope_table(ctx), rot_start=0, rotary_dim=self.position.rotary_dim,
            slots=group.slots, k_pages=store.k_pages, v_pages=store.v_pages, row_norm=True)
        if not ops.mixed_attention_mfma_ok(out.dtype, H, self.cache_dim, store.k_pages.shape[2]):
            ops.mixed_attention(q, d, out, e, store.k_pages, store.v_pages, group.block_table, ctx.seq_of_token, ctx.positions,
                                H, self.scale, self.talk, self.softcap, self.window or 0, out_scale)
            return
        single, portions = self._items(ctx, out.device)
        ops.mixed_attention_mfma(q, d, out, e, store.k_pages, store.v_pages, group.block_table, single, portions,
                                 ctx.graph_capacity or ctx.max_kv_len, H, self.scale, self.talk, self.softcap,
                                 self.window or 0, out_scale, self.talk_low)

    @staticmethod
    def _items(ctx: Any, device: Any):
        """The step's items for the matrix-core kernels, shared by the layers."""
        plan = ctx.scratch.get("mixed_attention_items")
        if plan is None:
            if ctx.seq_records is not None and ctx.max_q_len == 1:
                # every sequence is one token: its records are in the step's buffer already (and are refreshed with it
                # when the step is a replayed graph)
                plan = (ctx.seq_records, None)
            else:
                single, portions = ops.mixed_attention_items(ctx.q_lens, ctx.q_start_host, ctx.n_cached)
                both = ops.upload(np.concatenate([single, portions]), torch.int32, device)
                plan = (both[: len(single)] if len(single) else None, both[len(single) :] if len(portions) else None)
            ctx.scratch["mixed_attention_items"] = plan
        return plan


register_part("mixer", "mixed_attention", MixedAttention)
