"""Mixers whose memory is a matrix per head with one decay per token and head (``ops.matrix_memory``).

``gated_delta_rule``  q = W_q h and k = W_k h (``kv_heads`` x ``key_dim``), v = W_v h (``heads`` x ``value_dim``); each passes a
    short causal convolution over time per channel and silu; q and k are divided by their lengths per head, q times
    key_dim^(-1/2).  With b = sigmoid(W_b h) and g = exp(-exp(A_log) softplus(W_a h + dt_bias)) per head:
    S <- g S, u = b (v - S^T k), S <- S + k u^T, o = S^T q.  Every head's o over its root mean square times a gain shared by the
    heads, times silu(W_g h), then W_o.
``exp_gated_memory``  q = W_q h key_dim^(-1/2), k = W_k h, v = W_v h; log gates i = cap tanh((W_i h + b_i) / cap) and f = log
    sigmoid(cap tanh((W_f h + b_f) / cap)) per head, kept over e^m with m <- max(f + m, i) from zero: S <- e^(f + m' - m) S +
    e^(i - m) k v^T, n the same with k alone, o = S^T q / (max(|n . q|, e^-m) + 1e-6).  Every head's o over its root mean square,
    times a gain per column, times sigmoid(W_g h), then W_o.

What a request keeps between steps is one float32 row per slot: the convolution's last inputs and the heads' memories, or
the memories, the normalisers n and the m.  The projections leave float32 rows also where the model computes in bfloat16,
so everything that enters the recurrence is 32-bit.
"""
from __future__ import annotations

from typing import Dict, List, Optional

import numpy as np
import torch

from ..kernels import ops
from .base import LayerCache, Mixer, PartEnv, StateNeed, StepContext, StepPlan, StepShape, WeightDecl, register_part
from .linear import linear, linear_into_stream


def plan_memory_chunks(shape: StepShape) -> StepPlan:
    """The chunks of up to ``ops.MEMORY_CHUNK`` tokens every entry's tokens are cut into, (first token, tokens) each, an
    entry's side by side, and every entry's first.  A step of single tokens lists none."""
    items, entry_item, t0 = [], [], 0
    if any(n != 1 for n in shape.lens):
        for n in shape.lens:
            entry_item.append(len(items) // 2)
            for at in range(0, n, ops.MEMORY_CHUNK):
                items.extend((t0 + at, min(ops.MEMORY_CHUNK, n - at)))
            t0 += n
    return StepPlan(arrays={"items": np.asarray(items, dtype=np.int32), "entry_item": np.asarray(entry_item, dtype=np.int32)},
                    facts={"num_items": len(items) // 2})


class _MemoryMixer(Mixer):
    """What the two have in common: sizes, names, one input matrix whose columns are padded to whole 64-byte pieces."""
    DEFAULT_NAMES: Dict[str, str] = {}
    step_planners = {"memory chunks": plan_memory_chunks}

    def __init__(self, hidden_size: int, heads: int, kv_heads: int, key_dim: int, value_dim: int, norm_eps: float, prefix: str,
                 names: Optional[Dict[str, str]] = None):
        if min(heads, kv_heads, key_dim, value_dim) < 1 or heads % kv_heads:
            raise ValueError(f"{heads} heads over {kv_heads} key heads of sizes {key_dim} and {value_dim}")
        if key_dim > ops.MEMORY_MAX_KEYS:
            raise ValueError(f"{key_dim} key channels a head: at most {ops.MEMORY_MAX_KEYS}")
        self.hidden_size, self.heads, self.kv_heads, self.key_dim, self.value_dim = hidden_size, heads, kv_heads, key_dim, value_dim
        self.norm_eps, self.prefix = float(norm_eps), prefix
        self.names = {**self.DEFAULT_NAMES, **(names or {})}
        self.qk, self.inner = kv_heads * key_dim, heads * value_dim
        self.memory = heads * key_dim * value_dim        # values of a request's memories

    def _name(self, role: str) -> str:
        return f"{self.prefix}.{self.names[role]}"

    def kernel_families(self, dtype):
        return ("matrix_memory", "decay_scan")

    @staticmethod
    def _rows(cache: LayerCache) -> torch.Tensor:
        return cache.state.view(cache.state.shape[0], -1)

    def _input_rows(self):
        """(role, rows) of the input matrix, in order."""
        raise NotImplementedError

    def _input_decls(self) -> List[WeightDecl]:
        out, off = [], 0
        for role, n in self._input_rows():
            out.append(WeightDecl(self._name(role), (n, self.hidden_size), merged_into=f"{self.prefix}.in", row_offset=off))
            off += n
        return out

    def _bind_input(self, tensors: Dict[str, torch.Tensor]) -> None:
        w = tensors[f"{self.prefix}.in"]
        pad = -w.shape[0] % 16
        self.w_in = (torch.cat((w, w.new_zeros((pad, self.hidden_size)))) if pad else w).contiguous()
        self.at, off = {}, 0
        for role, n in self._input_rows():
            self.at[role] = slice(off, off + n)
            off += n


@register_part("mixer", "gated_delta_rule")
class GatedDeltaRule(_MemoryMixer):
    DEFAULT_NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "b": "b", "a": "a", "q_conv": "q.conv", "k_conv": "k.conv",
                     "v_conv": "v.conv", "a_log": "A_log", "dt_bias": "dt_bias", "norm": "norm", "o": "o"}

    def __init__(self, hidden_size: int, heads: int, kv_heads: int, key_dim: int, value_dim: int, conv: int, norm_eps: float,
                 prefix: str, names: Optional[Dict[str, str]] = None):
        super().__init__(hidden_size, heads, kv_heads, key_dim, value_dim, norm_eps, prefix, names)
        if not 1 <= conv <= ops.SHORT_CONV_MAX_TAPS:
            raise ValueError(f"a convolution of {conv} taps: 1 to {ops.SHORT_CONV_MAX_TAPS}")
        if value_dim > ops.MEMORY_MAX_KEYS:
            raise ValueError(f"{value_dim} value channels a head: at most {ops.MEMORY_MAX_KEYS}")
        self.taps, self.channels = int(conv), 2 * self.qk + self.inner
        # the memories lie ahead of the convolution's inputs: whole 16-byte pieces wherever their own sizes allow it
        self.carry = (self.taps - 1) * self.channels

    def cache_need(self):
        return StateNeed((self.memory + self.carry,), torch.float32, graph_safe=True)

    def _input_rows(self):
        return (("q", self.qk), ("k", self.qk), ("v", self.inner), ("g", self.inner), ("b", self.heads), ("a", self.heads))

    def weights(self) -> List[WeightDecl]:
        small = dict(keep_fp32=True)
        conv, off = [], 0
        for role, n in (("q_conv", self.qk), ("k_conv", self.qk), ("v_conv", self.inner)):
            conv.append(WeightDecl(self._name(role), (n, self.taps), merged_into=f"{self.prefix}.conv", row_offset=off, **small))
            off += n
        return self._input_decls() + conv + [
            WeightDecl(self._name("a_log"), (self.heads,), **small), WeightDecl(self._name("dt_bias"), (self.heads,), **small),
            WeightDecl(self._name("norm"), (self.value_dim,), init="gain", **small),
            WeightDecl(self._name("o"), (self.hidden_size, self.inner))]

    def bind(self, tensors: Dict[str, torch.Tensor], env: PartEnv) -> None:
        self._bind_input(tensors)
        get = lambda role: tensors[self._name(role)].contiguous()        # noqa: E731
        self.w_conv = tensors[f"{self.prefix}.conv"].t().contiguous()
        self.a_rate = torch.exp(get("a_log").to(torch.float64)).to(torch.float32).contiguous()
        self.dt_bias, self.gain, self.w_o = get("dt_bias"), get("norm"), get("o")

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: LayerCache) -> torch.Tensor:
        rows, at = self._rows(cache), self.at
        proj = linear(x, self.w_in, out_dtype=torch.float32)                        # q | k | v | g | b | a
        qkv, gates = ops.delta_prepare(proj[:, :self.channels], self.w_conv, proj[:, at["b"]], proj[:, at["a"]], self.a_rate,
                                       self.dt_bias, rows, self.memory, ctx, self.heads, self.kv_heads, self.key_dim, self.value_dim,
                                       self.key_dim ** -0.5, write_state=cache.owner)
        o, _ = ops.matrix_memory(qkv[:, at["q"]], qkv[:, at["k"]], qkv[:, at["v"]], gates[:, 0], gates[:, 1], ops.MEMORY_DELTA, rows, 0,
                                 ctx, self.heads, self.kv_heads, self.key_dim, self.value_dim, ctx.plans["memory chunks"], write_state=cache.owner)
        y = ops.gated_unit_norm(o, proj[:, at["g"]], self.gain, self.norm_eps, self.heads, ops.GATE_SILU, ctx.dtype)
        return linear_into_stream(y, self.w_o, ctx)


@register_part("mixer", "exp_gated_memory")
class ExpGatedMemory(_MemoryMixer):
    DEFAULT_NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "i": "i", "f": "f", "i_bias": "i.b", "f_bias": "f.b", "norm": "norm",
                     "o": "o"}

    def __init__(self, hidden_size: int, heads: int, key_dim: int, value_dim: int, gate_cap: float, norm_eps: float, prefix: str,
                 names: Optional[Dict[str, str]] = None):
        super().__init__(hidden_size, heads, heads, key_dim, value_dim, norm_eps, prefix, names)
        if not gate_cap > 0:
            raise ValueError("gate_cap must be positive")
        self.cap = float(gate_cap)
        self.norm_at = self.memory                       # a request's row: memories | normalisers | running maxima
        self.m_at = self.norm_at + self.qk

    def cache_need(self):
        return StateNeed((self.m_at + self.heads,), torch.float32, graph_safe=True)

    def _input_rows(self):
        return (("q", self.qk), ("k", self.qk), ("v", self.inner), ("g", self.inner), ("i", self.heads), ("f", self.heads))

    def weights(self) -> List[WeightDecl]:
        small = dict(keep_fp32=True)
        return self._input_decls() + [
            WeightDecl(self._name("i_bias"), (self.heads,), **small), WeightDecl(self._name("f_bias"), (self.heads,), **small),
            WeightDecl(self._name("norm"), (self.inner,), init="gain", **small),
            WeightDecl(self._name("o"), (self.hidden_size, self.inner))]

    def bind(self, tensors: Dict[str, torch.Tensor], env: PartEnv) -> None:
        self._bind_input(tensors)
        get = lambda role: tensors[self._name(role)].contiguous()        # noqa: E731
        self.b_i, self.b_f, self.gain, self.w_o = get("i_bias"), get("f_bias"), get("norm"), get("o")

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: LayerCache) -> torch.Tensor:
        rows, at = self._rows(cache), self.at
        proj = linear(x, self.w_in, out_dtype=torch.float32)                        # q | k | v | g | i | f
        gates = ops.exp_gates(proj[:, at["i"]], proj[:, at["f"]], self.b_i, self.b_f, self.cap, rows, self.m_at, ctx,
                              write_state=cache.owner)
        o, norm = ops.matrix_memory(proj[:, at["q"]], proj[:, at["k"]], proj[:, at["v"]], gates[:, 0], gates[:, 1], ops.MEMORY_SUM, rows,
                                    0, ctx, self.heads, self.heads, self.key_dim, self.value_dim, ctx.plans["memory chunks"], q_scale=self.key_dim ** -0.5,
                                    norm_off=self.norm_at, write_state=cache.owner)
        y = ops.gated_unit_norm(o, proj[:, at["g"]], self.gain, self.norm_eps, self.heads, ops.GATE_SIGMOID, ctx.dtype, den=norm,
                                least=gates[:, 2])
        return linear_into_stream(y, self.w_o, ctx)
