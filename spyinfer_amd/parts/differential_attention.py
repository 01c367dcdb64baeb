"""Differential attention over the paged cache: every head has two maps, each a softmax attention of its own with queries
and keys of ``dim`` values, over the same values; the head's result is a1 - lam a2 with one number lam for the layer,
lam = exp(lq1 . lk1) - exp(lq2 . lk2) + diff, then over its root mean square (no weight) and times 1 - diff; then the output
projection.  Queries and keys are normed per head and map (one weight for all) and rotated by angles formed in the kernel.

What is cached per token and kv head: ONE key row [map 1 | map 2] and one value row.  The queries of a head are two rows,
[q1 | 0] and [0 | q2], in the group of their kv head, so the attention kernels see a head count of two per head and read
keys and values once for both maps.  A layer with ``own_kv`` False has no projections of keys and values and reads the
cache of another layer (run order: ``LayerCall(layer, cache=that layer's, store=False)``).
"""
from __future__ import annotations

import math
from typing import Optional

import torch

from ..kernels import ops
from ..weights.loader import WeightSpec
from .attention import PagedAttention, attention_meta
from .base import PositionEncoding

MAPS = 2


class DifferentialAttention(PagedAttention):
    def __init__(self, hidden_size: int, heads: int, kv_heads: int, dim: int, value_dim: int, position: Optional[PositionEncoding],
                 scale: float, norm_eps: float, diff: float, own_kv: bool = True, names: Optional[dict] = None):
        """``diff``: the constant of lam and of the result's factor.  ``names``: tensor names behind the prefix for q, k, v, o,
        q_norm, k_norm, lq1, lk1, lq2, lk2."""
        if heads % kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        # (what plans tiles and asks for the cache sees two query heads a head)
        super().__init__(hidden_size, MAPS * heads, kv_heads, dim, position, qk_norm_eps=norm_eps, scale=scale, value_dim=value_dim,
                         names=dict(dict(lq1=".lq1", lk1=".lk1", lq2=".lq2", lk2=".lk2"), **(names or {})), formed_angles=True)
        self.heads, self.diff, self.own_kv = heads, float(diff), bool(own_kv)
        self.head_dim = -(-max(MAPS * dim, value_dim) // 16) * 16
        self.lam = None

    def weight_specs(self, prefix):
        H, h, g, dk, dv, n = self.hidden_size, self.heads, self.num_kv_heads, self.key_dim, self.value_dim, self.names
        specs = [WeightSpec(prefix + n["q"], (h * MAPS * dk, H)), WeightSpec(prefix + n["o"], (H, h * dv)), WeightSpec(prefix + n["q_norm"], (dk,), "norm")]
        if self.own_kv:
            specs += [WeightSpec(prefix + n["k"], (g * MAPS * dk, H)), WeightSpec(prefix + n["v"], (g * dv, H)), WeightSpec(prefix + n["k_norm"], (dk,), "norm")]
        return specs + [WeightSpec(prefix + n[x], (dk,), "bias") for x in ("lq1", "lk1", "lq2", "lk2")]

    def bind(self, prefix, weights):
        n = self.names
        mats = [weights.pop(prefix + n[c]) for c in ("qkv" if self.own_kv else "q")]
        if len({m.dtype for m in mats}) > 1:
            mats = [m.float() for m in mats]
        self.w_qkv, self.w_qkv_tiled = ops.weight_forms(torch.cat(mats, dim=0).contiguous())
        del mats
        self.w_o, self.w_o_tiled = ops.weight_forms(weights.pop(prefix + n["o"]))
        self.q_norm = weights[prefix + n["q_norm"]]
        self.k_norm = weights[prefix + n["k_norm"]] if self.own_kv else None
        if self.own_kv and self.q_norm.dtype != self.k_norm.dtype:
            self.q_norm, self.k_norm = self.q_norm.float(), self.k_norm.float()
        # one number for the layer, formed once
        dot = lambda a, b: float((weights[prefix + n[a]].double() * weights[prefix + n[b]].double()).sum())
        self.lam = math.exp(dot("lq1", "lk1")) - math.exp(dot("lq2", "lk2")) + self.diff
        if self.position is not None:
            self.position.prepare(self.w_o.device, 0)

    def forward(self, x, batch, cache, store=True):
        if store and not self.own_kv:
            raise ValueError("a layer without keys and values of its own reads another layer's cache")
        nq, nkv, d = self.num_heads, self.num_kv_heads, self.head_dim
        qkv = ops.linear_few(x, self.w_qkv, self.w_qkv_tiled)
        freq, mag, rdim = self.position.frequencies() if self.position is not None else (None, 1.0, 0)
        if mag != 1.0:
            raise ValueError("a rotation with a factor on cos and sin is not implemented here")
        meta = attention_meta(batch, cache.group, nq // nkv, self._big_rows(batch, cache.page_size))
        slots = batch.slot_mapping(cache.group) if store else None
        q = ops.norm_rope_store(qkv, self.heads, nkv, self.key_dim, self.value_dim, d, self.q_norm, self.k_norm, self.qk_norm_eps, freq, rdim,
                                batch.positions, cache.k, cache.v, cache.page_size, slots, maps=MAPS, interleaved=self._pairs_interleaved())
        a = ops.paged_attention(q, cache.k, cache.v, cache.page_size, meta, nq, nkv, d, self.scale, None)
        y = ops.map_difference(a, self.heads, self.value_dim, d, self.lam, self.qk_norm_eps, 1.0 - self.diff)
        return ops.linear_few(y, self.w_o, self.w_o_tiled)
