"""Risolorn as a plan.  Every layer is a parallel block: one elementwise squashing (tanh with a learned slope, gain and
shift) whose output both the mixer and the routed feed-forward read, and their sum added to the stream.  Mixers: the gated
delta rule behind short convolutions, a matrix memory with exponential gates, or grouped-query attention with biases, a
stretched rotation of adjacent pairs, sinks, and keys of the query's own chunk alone.  Feed-forwards: experts scored by
sigmoids, chosen by score + correction from the groups whose two best choice scores sum highest, weighed by their scores as
they are.  The head is a matrix of its own, its logits times a scale.
Tensor names: ``embed``, ``head``, ``l<i>.norm1 (.alpha, .b)``, ``l<i>.mix.q / k / v (.conv) / g / b / a / A_log / dt_bias / norm / o``
(delta), ``l<i>.mix.q / k / v / g / i / f (.b) / norm / o`` (mlstm), ``l<i>.mix.q / k / v (.b) / sink / o`` (attention),
``l<i>.mlp.router / correction / e<j>.gate|up|down``, ``final.norm``.
"""
from __future__ import annotations

from ..config.model_config import RisolornConfig, RisolornDelta, RisolornMemory
from .model import Choice, ModelPlan
from .registry import register_architecture

ATTENTION_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_bias": "q.b", "k_bias": "k.b", "v_bias": "v.b", "sink": "sink"}


def _mixer(m, prefix: str, H: int, eps: float) -> Choice:
    if isinstance(m, RisolornDelta):
        return Choice("mixer", "gated_delta_rule", dict(
            hidden_size=H, heads=m.heads, kv_heads=m.kv_heads, key_dim=m.dim, value_dim=m.vdim, conv=m.conv, norm_eps=eps, prefix=prefix))
    if isinstance(m, RisolornMemory):
        return Choice("mixer", "exp_gated_memory", dict(
            hidden_size=H, heads=m.heads, key_dim=m.dim, value_dim=m.vdim, gate_cap=m.gate_cap, norm_eps=eps, prefix=prefix))
    position = None
    if m.rot_dims:
        sc = m.rot_scaling
        position = Choice("position", "rotary", dict(
            head_dim=m.dim, theta=m.rot_base, rotary_dim=m.rot_dims, pairing="adjacent", max_positions=None, exact=True,
            scaling=None if sc is None else (sc.factor, sc.original, sc.fast, sc.slow)))
    return Choice("mixer", "gqa_attention", dict(
        hidden_size=H, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim, value_dim=m.vdim, prefix=prefix,
        position=position, bias=True, chunk=m.chunk, scale=m.scale, sink=True, names=ATTENTION_NAMES))


def risolorn_plan(cfg: RisolornConfig) -> ModelPlan:
    H, eps = cfg.hidden_size, cfg.norm_eps
    norm = lambda name: Choice("norm", "dynamic_tanh", dict(size=H, weight_name=name))      # noqa: E731
    layers = []
    for i, L in enumerate(cfg.layers):
        p, f = f"l{i}", L.mlp
        params = dict(norm=norm(f"{p}.norm1"), mixer=_mixer(L.mixer, f"{p}.mix", H, eps))
        if f is not None:
            params["ffn"] = Choice("ffn", "routed_experts", dict(
                hidden_size=H, experts=f.experts, intermediate_size=f.ff, top=f.top, limit=None, prefix=f"{p}.mlp", routing="sigmoid",
                correction=True, renormalize=False, groups=f.groups, keep_groups=f.keep, group_top=2))
        layers.append(Choice("block", "parallel", params))
    return ModelPlan(
        vocab_size=cfg.vocab_size, hidden_size=H, embedding_weight="embed", layers=layers, final_norm=norm("final.norm"),
        head_weight="head", embedding_scale=cfg.embedding_scale, logit_scale=cfg.logit_scale, init_std=0.05)


register_architecture("Risolorn", RisolornConfig.from_dict, risolorn_plan)
