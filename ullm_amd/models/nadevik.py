"""Nadevik as a plan.  Every layer norms what its sublayers put out and nothing else: x += norm(mixer(x + conv(x))),
x += norm(experts(x)), with RMS norms whose gains are stored around zero and a short convolution over time ahead of
the mixer.  Mixers: two side by side on the same input, grouped-query attention without positions (convolved q, k and
v, norms over the whole projections, soft-capped scores, sigmoid weights, a window and beyond it one key per block of
tokens) and a selective scan with a state per channel, added with two weights; or latent attention with a window,
whose keys another layer's may be.  Feed-forwards: experts chosen from the best groups and weighed by their softmax
scores as they are.  The embedding is a scaled table plus a hashed bigram table; the head is the embedding table.
Tensor names: ``embed``, ``bigram``, ``l<i>.norm1 / norm2 / canon1``, ``l<i>.mix.left.q / k / v (.conv, q.norm, k.norm) /
pb / o``, ``l<i>.mix.right.in / conv / conv.b / x / dt / dt.b / A_log / D / o``, ``l<i>.mix.q / dkv / dkv.norm / uk / uv / g /
o``, ``l<i>.mlp.router / e<j>.gate|up|down``, ``final.norm``.
"""
from __future__ import annotations

from ..config.model_config import NadevikConfig, NadevikParallel
from .model import Choice, ModelPlan
from .registry import register_architecture

ATTENTION_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm", "q_conv": "q.conv",
                   "k_conv": "k.conv", "v_conv": "v.conv", "bias": "pb"}


def _mixer(m, prefix: str, H: int, eps: float) -> Choice:
    if isinstance(m, NadevikParallel):
        a, r = m.left, m.right
        left = Choice("mixer", "pooled_attention", dict(
            hidden_size=H, num_heads=a.heads, num_kv_heads=a.kv_heads, head_dim=a.dim, value_dim=a.vdim, taps=a.conv,
            window=a.window, pool=a.pool, scale=a.scale, softcap=a.softcap, norm_eps=eps, prefix=f"{prefix}.left",
            names=ATTENTION_NAMES))
        right = Choice("mixer", "selective_scan", dict(hidden_size=H, inner=r.inner, state=r.state, dt_rank=r.dt_rank,
                                                       conv=r.conv, prefix=f"{prefix}.right"))
        return Choice("mixer", "side_by_side", dict(left=left, right=right, left_scale=m.left_scale, right_scale=m.right_scale))
    position = None
    if m.rot_dim:
        position = Choice("position", "rotary", dict(head_dim=m.rot_dim, theta=m.rot_base, pairing="adjacent", exact=True))
    return Choice("mixer", "latent_attention", dict(
        hidden_size=H, num_heads=m.heads, head_dim=m.dim, rot_dim=m.rot_dim, value_dim=m.vdim, q_rank=None, kv_rank=m.kv_rank,
        scale=m.scale, norm_eps=eps, prefix=prefix, position=position, window=m.window, own_kv=m.kv_from is None,
        head_gate=False, value_gate=True, names={"uq": "q"}))


def nadevik_plan(cfg: NadevikConfig) -> ModelPlan:
    H, eps = cfg.hidden_size, cfg.norm_eps
    norm = lambda name: Choice("norm", "rmsnorm", dict(size=H, eps=eps, weight_name=name, around_zero=True))      # noqa: E731
    layers, kv_from, unused = [], {}, []
    for i, L in enumerate(cfg.layers):
        p = f"l{i}"
        params = dict(hidden_size=H, mixer=_mixer(L.mixer, f"{p}.mix", H, eps), mixer_post=norm(f"{p}.norm1"),
                      conv_taps=cfg.canon_taps, conv_weight=f"{p}.canon1")
        f = L.mlp
        if f is None:
            unused.append(f"{p}.norm2")              # a file may hold it although the layer has no use for it
        else:
            params.update(ffn_post=norm(f"{p}.norm2"), ffn=Choice("ffn", "routed_experts", dict(
                hidden_size=H, experts=f.experts, intermediate_size=f.ff, top=f.top, limit=f.limit, prefix=f"{p}.mlp",
                correction=False, renormalize=False, groups=f.groups, keep_groups=f.keep)))
        if getattr(L.mixer, "kv_from", None) is not None:
            kv_from[i] = L.mixer.kv_from
        layers.append(Choice("block", "postnorm", params))
    embedder = Choice("embedding", "table_sum", dict(
        vocab_size=cfg.vocab_size, hidden_size=H, weight_name="embed", scale=cfg.embedding_scale,
        pair_weight_name="bigram" if cfg.bigram_buckets else None, pair_buckets=cfg.bigram_buckets,
        pair_mul_prev=cfg.bigram_mul_prev, pair_mul_cur=cfg.bigram_mul_cur))
    return ModelPlan(
        vocab_size=cfg.vocab_size, hidden_size=H, embedding_weight="embed", layers=layers, final_norm=norm("final.norm"),
        head_weight="head", tie_head_to_embedding=True, embedder=embedder, kv_from=kv_from, unused_tensors=tuple(unused),
        init_std=0.05)


register_architecture("Nadevik", NadevikConfig.from_dict, nadevik_plan)
