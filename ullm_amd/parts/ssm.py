"""Selective state-space mixers over per-request state.

``mamba2``, the Mamba-2 form:

The input projection's rows are z | x | B | C | dt (z, x: heads * head_dim; B, C: groups * state; dt: heads).
x | B | C pass a short causal convolution per channel and silu; dt = softplus(dt + dt_bias).  Per head h
(its B and C are those of group h // (heads / groups)) the state S [state, head_dim] moves token by token,
S = exp(-exp(A_log_h) dt) S + dt B x^T, and y = S^T C + D_h x.  y * silu(z) is RMS-normed in ``norm_groups``
equal parts, multiplied by a gain and projected out.

What a request keeps between steps is one float32 row per slot: the convolution's last taps-1 inputs, then
every head's state.  Everything behind the input projection is 32-bit (the projection leaves float32 rows
also where the model computes in bfloat16); the recurrence walks an entry's tokens in order whatever the
batch holds, so a token's result does not depend on how its prompt was cut.

``selective_scan``, the first Mamba form, with a state per channel:

The input projection's rows are x | z (``inner`` each).  x passes the short convolution (with a bias) and silu; W_x x is
dt | B | C (``dt_rank``, ``state``, ``state`` values); the step sizes are softplus(W_dt dt + bias), one per channel.  Per
channel c and state n:  S = exp(-exp(A_log) dt) S + dt x B,  y = sum_n S C + D x;  y * silu(z) is projected out.  A
request's float32 row holds the convolution's last inputs, then the states.  Step sizes, decays and states are 32-bit;
the projections and the convolution's result are stored in the compute dtype (the step sizes' last product in 32-bit).
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import numpy as np
import torch

from ..kernels import ops
from .base import LayerCache, Mixer, PartEnv, StateNeed, StepContext, StepPlan, StepShape, WeightDecl, register_part
from .linear import linear, linear_into_stream

DEFAULT_NAMES = {"in": "in_proj.weight", "conv": "conv1d.weight", "conv_bias": "conv1d.bias", "dt_bias": "dt_bias",
                 "a_log": "A_log", "d": "D", "norm": "norm.weight", "out": "out_proj.weight"}


@register_part("mixer", "mamba2")
class Mamba2(Mixer):
    def __init__(self, hidden_size: int, heads: int, head_dim: int, state: int, groups: int, conv: int,
                 norm_groups: int, norm_eps: float, prefix: str, names: Optional[Dict[str, str]] = None):
        if heads % groups:
            raise ValueError(f"{heads} heads are not a multiple of {groups} groups")
        if (heads * head_dim) % norm_groups:
            raise ValueError(f"{heads * head_dim} inner values do not cut into {norm_groups} equal parts")
        if not 1 <= conv <= ops.CONV_MAX_TAPS:
            raise ValueError(f"a convolution of {conv} taps: 1 to {ops.CONV_MAX_TAPS}")
        self.hidden_size, self.heads, self.head_dim, self.state, self.groups = hidden_size, heads, head_dim, state, groups
        self.taps, self.norm_groups, self.norm_eps, self.prefix = conv, norm_groups, float(norm_eps), prefix
        self.names = {**DEFAULT_NAMES, **(names or {})}
        self.inner = heads * head_dim
        self.channels = self.inner + 2 * groups * state              # x | B | C
        self.carry = (conv - 1) * self.channels                       # the convolution's part of the state row

    def _name(self, role: str) -> str:
        return f"{self.prefix}.{self.names[role]}"

    def cache_need(self):
        return StateNeed((self.carry + self.heads * self.state * self.head_dim,), torch.float32, graph_safe=True)

    def weights(self) -> List[WeightDecl]:
        H, small = self.hidden_size, dict(keep_fp32=True)
        return [WeightDecl(self._name("in"), (self.inner + self.channels + self.heads, H)),
                WeightDecl(self._name("conv"), (self.channels, self.taps), **small),
                WeightDecl(self._name("conv_bias"), (self.channels,), **small),
                WeightDecl(self._name("dt_bias"), (self.heads,), **small),
                WeightDecl(self._name("a_log"), (self.heads,), **small),
                WeightDecl(self._name("d"), (self.heads,), **small),
                WeightDecl(self._name("norm"), (self.inner,), init="gain", **small),
                WeightDecl(self._name("out"), (H, self.inner))]

    def bind(self, tensors: Dict[str, torch.Tensor], env: PartEnv) -> None:
        get = lambda role: tensors[self._name(role)].contiguous()       # noqa: E731
        self.w_in, self.w_out = get("in"), get("out")
        self.conv_w, self.conv_b = get("conv"), get("conv_bias")
        self.dt_bias, self.a_log, self.d_skip, self.norm_gain = get("dt_bias"), get("a_log"), get("d"), get("norm")

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: LayerCache) -> torch.Tensor:
        proj = linear(x, self.w_in, out_dtype=torch.float32)             # z | x | B | C | dt
        rows = cache.state.view(cache.state.shape[0], -1)
        xbc = ops.conv_silu(proj, self.inner, self.channels, self.conv_w, self.conv_b, rows, ctx.token_entry,
                            ctx.q_start, ctx.entry_slot, ctx.num_entries, update_carry=cache.owner)
        y = ops.ssm_scan(xbc, proj, self.inner + self.channels, self.dt_bias, self.a_log, self.d_skip, rows, self.carry,
                         ctx.q_start, ctx.entry_slot, ctx.num_entries, self.heads, self.groups, self.state,
                         self.head_dim, write_state=cache.owner)
        gated = ops.gated_group_norm(y, proj, 0, self.norm_gain, self.norm_eps, self.norm_groups, ctx.dtype)
        return linear_into_stream(gated, self.w_out, ctx)


def plan_scan_segments(shape: StepShape) -> StepPlan:
    """The segments of up to ``ops.SCAN_SEGMENT`` tokens an entry's tokens are cut into, as (entry, first token, tokens, what:
    0 its only one, 1 one of several, 2 the last of several), and for entries of several (entry, first item, items).  A step
    of single tokens lists none."""
    items, chains, t0 = [], [], 0
    if any(n != 1 for n in shape.lens):
        for b, n in enumerate(shape.lens):
            count = -(-n // ops.SCAN_SEGMENT)
            if count > 1:
                chains.extend((b, len(items) // 4, count))
            for i in range(count):
                first = i * ops.SCAN_SEGMENT
                items.extend((b, t0 + first, min(ops.SCAN_SEGMENT, n - first), 0 if count == 1 else 1 if i + 1 < count else 2))
            t0 += n
    return StepPlan(arrays={"items": np.asarray(items, dtype=np.int32), "chains": np.asarray(chains, dtype=np.int32)},
                    facts={"num_items": len(items) // 4, "num_chains": len(chains) // 3})


SCAN_NAMES = {"in": "in", "conv": "conv", "conv_bias": "conv.b", "x": "x", "dt": "dt", "dt_bias": "dt.b", "a_log": "A_log",
              "d": "D", "out": "o"}


@register_part("mixer", "selective_scan")
class SelectiveScan(Mixer):
    step_planners = {"scan segments": plan_scan_segments}

    def __init__(self, hidden_size: int, inner: int, state: int, dt_rank: int, conv: int, prefix: str,
                 names: Optional[Dict[str, str]] = None):
        if min(inner, state, dt_rank) < 1 or state > ops.SELECTIVE_SCAN_MAX_STATE:
            raise ValueError(f"sizes must be positive and the state at most {ops.SELECTIVE_SCAN_MAX_STATE}")
        if not 1 <= conv <= ops.SHORT_CONV_MAX_TAPS:
            raise ValueError(f"a convolution of {conv} taps: 1 to {ops.SHORT_CONV_MAX_TAPS}")
        self.hidden_size, self.inner, self.state, self.dt_rank, self.taps = hidden_size, inner, state, dt_rank, conv
        self.prefix, self.names = prefix, {**SCAN_NAMES, **(names or {})}
        self.carry = (conv - 1) * inner                               # the convolution's part of the state row

    def _name(self, role: str) -> str:
        return f"{self.prefix}.{self.names[role]}"

    def kernel_families(self, dtype):
        return ("short_conv", "selective_scan")

    def cache_need(self):
        return StateNeed((self.carry + self.inner * self.state,), torch.float32, graph_safe=True)

    def weights(self) -> List[WeightDecl]:
        H, n, small = self.hidden_size, self.inner, dict(keep_fp32=True)
        return [WeightDecl(self._name("in"), (2 * n, H)),
                WeightDecl(self._name("conv"), (n, self.taps), **small), WeightDecl(self._name("conv_bias"), (n,), **small),
                WeightDecl(self._name("x"), (self.dt_rank + 2 * self.state, n)),
                WeightDecl(self._name("dt"), (n, self.dt_rank)), WeightDecl(self._name("dt_bias"), (n,), **small),
                WeightDecl(self._name("a_log"), (n, self.state), **small), WeightDecl(self._name("d"), (n,), **small),
                WeightDecl(self._name("out"), (H, n))]

    def bind(self, tensors: Dict[str, torch.Tensor], env: PartEnv) -> None:
        get = lambda role: tensors[self._name(role)]                     # noqa: E731
        self.w_in, self.w_out = get("in").contiguous(), get("out").contiguous()
        self.w_conv, self.b_conv = get("conv").t().contiguous(), get("conv_bias").contiguous()
        # the low-rank step sizes' inner size and the row dt | B | C are padded with zeros to multiples of eight: whole
        # 16-byte pieces
        r, pad = self.dt_rank, -self.dt_rank % 8
        x, dt = get("x"), get("dt")
        self.w_x = torch.cat((x[:r], x.new_zeros((pad, self.inner)), x[r:], x.new_zeros((-2 * self.state % 8, self.inner)))).contiguous()
        self.rank8 = r + pad
        self.w_dt = torch.cat((dt, dt.new_zeros((self.inner, pad))), dim=1).contiguous()
        self.dt_bias, self.d_skip = get("dt_bias").contiguous(), get("d").contiguous()
        # A log2(e), rounded to 32-bit once: a decay is then one exponent of two
        self.a_log2 = (-torch.exp(get("a_log").to(torch.float64)) * math.log2(math.e)).to(torch.float32).contiguous()

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: LayerCache) -> torch.Tensor:
        n, rows = self.inner, cache.state.view(cache.state.shape[0], -1)
        proj = linear(x, self.w_in)                                      # x | z
        u = ops.short_conv(proj[:, :n], self.w_conv, self.b_conv, rows, 0, ctx, ops.CONV_SILU, ctx.dtype, write_state=cache.owner)
        low = linear(u, self.w_x)                                        # dt | B | C
        dt = linear(low[:, :self.rank8], self.w_dt, out_dtype=torch.float32)
        y = ops.selective_scan(u, dt, low[:, self.rank8:self.rank8 + 2 * self.state], proj[:, n:], self.a_log2, self.dt_bias, self.d_skip, rows, self.carry, ctx,
                               ctx.plans["scan segments"], write_state=cache.owner)
        return linear_into_stream(y, self.w_out, ctx)
