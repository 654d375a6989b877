"""Attention over a sliding window and, beyond it, over blocks of tokens seen as one key and value each, as a mixer.

Grouped-query attention without positions.  q, k and v pass a short causal convolution over time per channel right
behind their projections; q and k are then RMS-normed over the whole projection, all heads at once, with a gain per value.
Scores q . k * scale are soft-capped (``softcap``; 0: not) and a number per head is added; the weight of a visible key is
the sigmoid of that, and the weights are not normalised over the keys (``weights="softmax"``: the softmax instead).
A query sees the last ``window`` tokens, its own included.  The tokens are also counted off in blocks of ``pool`` from
position 0 on, and every block that has ended ahead of the query's window stands in with one row: its keys averaged and
its values averaged, from the rows in the pages.  ``pool`` 0: the window alone; ``window`` 0: every earlier token.

What a request keeps: the window's keys and values in pages (a page lives until neither the window nor the block being
filled needs it), the blocks' means in pages of their own with one row per block, and the convolution's last inputs in
one float32 row.
"""
from __future__ import annotations

import functools
from typing import Dict, List, Optional

import numpy as np
import torch

from ..kernels import ops
from .attention import GQAttention, plan_attention_step
from .base import KVNeed, LayerCache, PartEnv, StateNeed, StepContext, StepPlan, StepShape, WeightDecl, register_part
from .linear import linear, linear_into_stream

DEFAULT_CONV_NAMES = {"q_conv": "q_conv.weight", "k_conv": "k_conv.weight", "v_conv": "v_conv.weight", "bias": "score_bias"}


@functools.lru_cache(maxsize=None)
def block_planner(pool: int):
    """The planner that lists the blocks of ``pool`` tokens a step completes, as (entry, block) pairs (``blocks``); a step
    of single tokens lists none: there the kernel that writes a token's key sees to its block."""
    def plan_blocks(shape: StepShape) -> StepPlan:
        pairs = []
        if any(n != 1 for n in shape.lens):
            for b, (n, start) in enumerate(zip(shape.lens, shape.starts)):
                pairs.extend(x for block in range(start // pool, (start + n) // pool) for x in (b, block))
        return StepPlan(arrays={"blocks": np.asarray(pairs, dtype=np.int32)}, facts={"num_blocks": len(pairs) // 2})
    return plan_blocks


@register_part("mixer", "pooled_attention")
class PooledAttention(GQAttention):
    folds_norm = False
    hands_norm_ahead = False

    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int, taps: int, window: int, pool: int,
                 norm_eps: float, prefix: str, value_dim: Optional[int] = None, scale: Optional[float] = None,
                 softcap: float = 0.0, weights: str = "sigmoid", names: Optional[Dict[str, str]] = None):
        if weights not in ("sigmoid", "softmax"):
            raise ValueError(f"weights={weights!r}: 'sigmoid' or 'softmax'")
        if not 1 <= taps <= ops.SHORT_CONV_MAX_TAPS:
            raise ValueError(f"a convolution of {taps} taps: 1 to {ops.SHORT_CONV_MAX_TAPS}")
        if window < 0 or pool < 0 or (pool and not window):
            raise ValueError("pooled blocks need a window")
        super().__init__(hidden_size, num_heads, num_kv_heads, head_dim, prefix, qk_norm_eps=norm_eps, qk_norm="whole",
                         window=window, scale=scale, value_dim=value_dim, names={**DEFAULT_CONV_NAMES, **(names or {})})
        self.taps, self.pool, self.softcap, self.softmax = int(taps), int(pool), float(softcap), weights == "softmax"
        self.columns = (self.nq + 2 * self.nkv) * self.hd
        self.step_planners = {"attention": plan_attention_step}
        if self.pool:
            self.step_planners[f"blocks of {self.pool}"] = block_planner(self.pool)

    def kernel_families(self, dtype):
        return ("pooled", "attention_pooled") if dtype == torch.bfloat16 and not self.softmax else ("pooled",)

    def cache_need(self):
        needs = [KVNeed(self.nkv, self.hd, max(self.window, self.pool))]
        if self.pool:
            needs.append(KVNeed(self.nkv, self.hd, 0, tokens_per_row=self.pool))
        needs.append(StateNeed((max(1, (self.taps - 1) * self.columns),), torch.float32, graph_safe=True))
        return needs

    def weights(self) -> List[WeightDecl]:
        sizes = (("q_conv", self.nq * self.dim), ("k_conv", self.nkv * self.dim), ("v_conv", self.nkv * self.vdim))
        return (self._general_weights() + [WeightDecl(self._name(role), (n, self.taps), keep_fp32=True) for role, n in sizes]
                + [WeightDecl(self._name("bias"), (self.nq,), keep_fp32=True)])

    def bind(self, tensors: Dict[str, torch.Tensor], env: PartEnv) -> None:
        self._general_bind(tensors, env)

        def padded(role: str, heads: int, size: int) -> torch.Tensor:          # [heads * size, taps] -> [taps, heads * hd]
            w = tensors[self._name(role)].to(torch.float32).view(heads, size, self.taps)
            wide = w.new_zeros((heads, self.hd, self.taps))
            wide[:, :size] = w
            return wide.view(heads * self.hd, self.taps).t()
        self.w_conv = torch.cat((padded("q_conv", self.nq, self.dim), padded("k_conv", self.nkv, self.dim),
                                 padded("v_conv", self.nkv, self.vdim)), dim=1).contiguous()
        self.score_bias = tensors[self._name("bias")].to(torch.float32).contiguous()

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: LayerCache) -> torch.Tensor:
        views = cache.parts
        tokens, state = views[0], views[-1].state
        pooled = views[1] if self.pool else None
        group = ctx.groups[tokens.group]
        pooled_group = ctx.groups[pooled.group] if self.pool else None
        pk, pv = (pooled.k_pool, pooled.v_pool) if self.pool else (None, None)
        proj = linear(x, self.w_qkv)                                             # q | k | v
        q = ops.conv_norm_write(proj, self.w_conv, state.view(state.shape[0], -1), 0, self.q_gain, self.k_gain, self.qk_norm_eps,
                                self.nq * self.dim, self.nkv * self.dim, ctx, group, tokens.k_pool, tokens.v_pool, self.nq,
                                self.nkv, self.hd, self.pool, pooled_group, pk, pv)
        if self.pool:
            plan = ctx.plans[f"blocks of {self.pool}"]
            if plan.facts["num_blocks"]:
                ops.block_means(plan.arrays["blocks"], plan.facts["num_blocks"], group, pooled_group, tokens.k_pool, tokens.v_pool,
                                pk, pv, self.pool, self.nkv, self.hd)
        out = ops.pooled_attention(q, tokens.k_pool, tokens.v_pool, ctx, group, self.nq, self.nkv, self.hd, self.scale, self.window,
                                   ctx.plans["attention"], self.softcap, self.score_bias, self.pool, pooled_group, pk, pv,
                                   softmax=self.softmax)
        return linear_into_stream(out, self.w_o, ctx)

    def fusable(self, residual, ctx: StepContext) -> bool:
        return False
