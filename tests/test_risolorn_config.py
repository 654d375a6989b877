"""Risolorn without a GPU: the configuration reader and what it refuses, the plan it becomes (tensor names and shapes, what a
block keeps), a cache group whose pages return with their chunk, rotation tables, and the plain implementation's own pieces
against explicit loops."""
import copy
import math
import random

import pytest
import torch

import plain_risolorn as plain
from ullm_amd.cache.manager import CacheGroupSpec, CacheManager
from ullm_amd.config import ConfigError, RisolornConfig
from ullm_amd.models import build_model
from ullm_amd.parts import KVNeed, StateNeed, build_part, cache_needs_of
from ullm_amd.parts.position import Rotary

MOE = dict(kind="moe", router=dict(experts=9, top=3, groups=dict(count=3, keep=2)), expert=dict(ff=10))
SCALING = dict(factor=3.0, original=64, fast=8.0, slow=0.5)


def att(mlp=MOE, chunk=11, **more):
    m = dict(heads=6, kv_heads=2, dim=10, vdim=14, scale=0.3, mask=dict(size=chunk), rot=dict(base=200.0, dims=6, scaling=SCALING))
    m.update(more)
    return dict(type="attention", mlp=mlp, mixer=m)


def delta(mlp=MOE, **more):
    return dict(type="delta", mlp=mlp, mixer=dict(dict(heads=4, kv_heads=2, dim=6, vdim=10, conv=3), **more))


def mlstm(mlp=MOE, **more):
    return dict(type="mlstm", mlp=mlp, mixer=dict(dict(heads=3, dim=8, vdim=6, gate_cap=5.0), **more))


CFG = dict(architecture="Risolorn", vocab=70, width=24, norm=dict(eps=1e-4), embedding=dict(scale=2.0), logit_scale=0.6,
           layers=[mlstm(), att(), delta(), att(mlp=None), delta(mlp=None), mlstm(mlp=None)])


def changed(path, value):
    c = copy.deepcopy(CFG)
    at = c
    for k in path[:-1]:
        at = at[k]
    if value is KeyError:
        del at[path[-1]]
    else:
        at[path[-1]] = value
    return c


def test_the_plan_names_every_tensor_of_the_design_with_its_shape():
    cfg, model = build_model(CFG)
    assert isinstance(cfg, RisolornConfig) and cfg.num_hidden_layers == 6 and cfg.logit_scale == 0.6 and cfg.embedding_scale == 2.0
    decls = model.weight_decls()
    assert {d.name: tuple(d.shape) for d in decls} == plain.tensor_shapes(CFG)
    assert not [d for d in decls if d.alias_of is not None]             # the head is a matrix of its own
    assert model.plan.logit_scale == 0.6 and model.plan.embedding_scale == 2.0
    ffn = model.blocks[0].ffn
    assert (ffn.top, ffn.groups, ffn.keep_groups, ffn.group_top, ffn.raw) == (3, 3, 2, 2, True)


def test_what_the_layers_keep():
    _, model = build_model(CFG)
    groups, _, states = model.cache_layout()
    assert len(groups) == 1 and groups[0].chunk == 11 and groups[0].window == 0 and len(groups[0].layers) == 2
    assert groups[0].head_dim == 32 and groups[0].num_kv_heads == 2
    conv = 2 * (2 * 2 * 6 + 4 * 10)
    assert sorted(n.shape[0] for n in states.values()) == sorted(2 * [4 * 6 * 10 + conv] + 2 * [3 * 8 * 6 + 3 * 8 + 3])
    assert all(n.graph_safe and n.dtype == torch.float32 for n in states.values())
    assert [type(n) for n in cache_needs_of(model.blocks[1])] == [KVNeed] and [type(n) for n in cache_needs_of(model.blocks[2])] == [StateNeed]
    # layers with other chunks are other groups: their pages return at other times
    _, model = build_model(changed(("layers", 3, "mixer", "mask"), dict(size=7)))
    assert sorted(g.chunk for g in model.cache_layout()[0]) == [7, 11]
    _, model = build_model(changed(("layers", 3, "mixer", "mask"), None))
    assert sorted(g.chunk for g in model.cache_layout()[0]) == [0, 11]


def test_defaults():
    c = dict(architecture="Risolorn", vocab=30, width=8, norm=dict(eps=1e-5),
             layers=[dict(type="attention", mixer=dict(heads=2, kv_heads=1, dim=4, scale=0.5), mlp=None),
                     dict(type="delta", mixer=dict(heads=2, kv_heads=2, dim=4, conv=1), mlp=dict(kind="moe", router=dict(experts=3, top=3), expert=dict(ff=4)))])
    cfg, model = build_model(c)
    a, f = cfg.layers[0].mixer, cfg.layers[1].mlp
    assert (a.vdim, a.chunk, a.rot_dims, cfg.logit_scale, cfg.embedding_scale, f.groups, f.keep) == (4, 0, 0, 1.0, 1.0, 1, 1)
    assert {d.name: tuple(d.shape) for d in model.weight_decls()} == plain.tensor_shapes(c)


@pytest.mark.parametrize("path,value", [
    (("layers",), []), (("layers", 0, "type"), "gla"), (("layers", 0, "mixer"), None), (("layers", 1, "mixer", "kv_heads"), 4),
    (("layers", 1, "mixer", "rot", "dims"), 5), (("layers", 1, "mixer", "rot", "dims"), 12), (("layers", 1, "mixer", "mask", "size"), -1),
    (("layers", 1, "mixer", "rot", "scaling"), 3), (("layers", 1, "mixer", "rot", "scaling", "factor"), 0.0), (("layers", 1, "mixer", "rot", "base"), 1.0),
    (("layers", 1, "mixer", "rot", "scaling"), dict(factor=2.0)), (("layers", 2, "mixer", "kv_heads"), 3), (("layers", 2, "mixer", "conv"), 0),
    (("layers", 2, "mixer", "conv"), KeyError), (("layers", 0, "mixer", "gate_cap"), 0.0), (("layers", 0, "mixer", "gate_cap"), KeyError),
    (("layers", 0, "mixer", "kv_heads"), 1), (("layers", 0, "mixer", "dim"), 0), (("layers", 0, "mlp", "kind"), "dense"),
    (("layers", 0, "mlp", "router", "groups", "count"), 4), (("layers", 0, "mlp", "router", "groups", "keep"), 4),
    (("layers", 0, "mlp", "router", "top"), 7), (("layers", 0, "mlp", "expert", "ff"), 0), (("vocab",), KeyError), (("norm",), {})])
def test_configurations_that_are_refused(path, value):
    with pytest.raises(ConfigError):
        RisolornConfig.from_dict(changed(path, value))


def test_parts_refuse_what_they_cannot_compute():
    base = dict(hidden_size=8, num_heads=2, num_kv_heads=1, head_dim=4, prefix="x")
    with pytest.raises(ValueError):
        build_part("mixer", "gqa_attention", window=4, chunk=4, **base)
    with pytest.raises(ValueError):
        build_part("mixer", "gqa_attention", chunk=-1, **base)
    with pytest.raises(ValueError):
        build_part("ffn", "routed_experts", hidden_size=8, experts=4, intermediate_size=4, top=1, limit=None, prefix="x", group_top=3)
    with pytest.raises(ValueError):
        build_part("mixer", "gated_delta_rule", hidden_size=8, heads=2, kv_heads=1, key_dim=4, value_dim=4, conv=17, norm_eps=1e-5, prefix="x")
    with pytest.raises(ValueError):
        build_part("mixer", "exp_gated_memory", hidden_size=8, heads=2, key_dim=513, value_dim=4, gate_cap=1.0, norm_eps=1e-5, prefix="x")


@pytest.mark.parametrize("dims,base,scaling", [(6, 200.0, (3.0, 64.0, 8.0, 0.5)), (16, 1e4, (8.0, 4096.0, 32.0, 1.0)), (2, 50.0, (4.0, 40.0, 2.0, 2.0)),
                                               (8, 1e6, (1.0, 100.0, 4.0, 1.0)), (64, 1e4, (2.0, 10.0, 1e6, 1e5)), (8, 500.0, None)])
def test_stretched_angles(dims, base, scaling):
    """The table against the formula: a ramp of no width, of all pairs, one that lies past the last pair."""
    d = None if scaling is None else dict(zip(("factor", "original", "fast", "slow"), scaling))
    freq, size = plain.rotation(dims, base, d)
    table = Rotary.make_table(dims, base, 3000, scaling=scaling, exact=True)
    for p in (0, 1, 77, 2999):
        for i in range(dims // 2):
            assert abs(table[p, i].item() - size * math.cos(p * freq[i])) < 2e-7
            assert abs(table[p, dims // 2 + i].item() - size * math.sin(p * freq[i])) < 2e-7


# ----------------------------------------------------------------------------- the cache

@pytest.mark.parametrize("chunk", [1, 3, 4, 6, 10, 16, 50])
def test_pages_return_when_their_chunk_is_over(chunk):
    m = CacheManager([CacheGroupSpec(2, 16, 0, (0,)), CacheGroupSpec(2, 16, 0, (1,), chunk=chunk)], [24, 24], page_size=4, max_requests=2)
    rc = m.admit("a")
    rng = random.Random(chunk)
    while rc.num_computed < 80:
        n = rng.choice([1, 1, 2, 7])
        assert m.reserve(rc, n)
        m.commit(rc, n)
        held = {i for i, p in enumerate(rc.tables[1]) if p >= 0}
        # the next query sees from its chunk's start on: those pages are held, pages wholly before it are not
        start = rc.num_computed // chunk * chunk
        assert held == set(range(start // 4, -(-rc.num_computed // 4))), (rc.num_computed, held)
        m.check()
    m.release(rc)
    assert m.num_free_pages(0) == 24 and m.num_free_pages(1) == 24


def test_no_prefixes_are_shared_with_chunks():
    m = CacheManager([CacheGroupSpec(2, 16, 0, (0,), chunk=8)], [8], page_size=4, max_requests=1, enable_prefix_cache=True)
    assert m.prefix_tree is None


# ----------------------------------------------------------------------------- the plain implementation itself

def test_plain_recurrences_against_loops_over_single_numbers():
    g = torch.Generator().manual_seed(1)
    T, N, P = 5, 3, 2
    q, k, v = (torch.randn(T, n, generator=g).double() for n in (N, N, P))
    keep, beta = torch.rand(T, generator=g).double(), torch.rand(T, generator=g).double()
    got = plain.delta_rule(q, k, v, keep, beta)
    S = [[0.0] * P for _ in range(N)]
    for t in range(T):
        for p in range(P):
            for n in range(N):
                S[n][p] *= keep[t].item()
            err = v[t, p].item() - sum(S[n][p] * k[t, n].item() for n in range(N))
            for n in range(N):
                S[n][p] += k[t, n].item() * beta[t].item() * err
            assert abs(got[t, p].item() - sum(S[n][p] * q[t, n].item() for n in range(N))) < 1e-12
    i, f = 3 * torch.randn(T, generator=g).double(), -torch.rand(T, generator=g).double()
    got = plain.exp_gated_memory(q, k, v, i, f)
    for t in range(T):
        # without the running maximum: every token's weight at t, and the maximum as the largest of the decayed gates and of
        # the decayed zero it starts from
        w = [math.exp(i[s].item() + f[s + 1:t + 1].sum().item()) for s in range(t + 1)]
        m = max([f[:t + 1].sum().item()] + [i[s].item() + f[s + 1:t + 1].sum().item() for s in range(t + 1)])
        kq = [(k[s] @ q[t]).item() for s in range(t + 1)]
        n = sum(a * b for a, b in zip(w, kq)) * math.exp(-m)
        for p in range(P):
            top = sum(a * b * v[s, p].item() for s, (a, b) in enumerate(zip(w, kq))) * math.exp(-m)
            assert abs(got[t, p].item() - top / (max(abs(n), math.exp(-m)) + 1e-6)) < 1e-9


def test_plain_masks_choice_and_convolution_against_loops():
    g = torch.Generator().manual_seed(2)
    for T, size in ((23, 5), (9, 1), (8, 20), (12, 0)):
        seen = plain.same_chunk(T, size)
        for i in range(T):
            assert torch.nonzero(seen[i]).flatten().tolist() == [j for j in range(i + 1) if not size or j // size == i // size]
    c = torch.tensor([0.1, 0.5, 0.45, 0.3, 0.6, -0.9]).double()            # groups (0 1), (2 3), (4 5): sums 0.6, 0.75, -0.3
    assert plain.choose_experts(c, 3, 3, 2)[0] == [1, 2, 3]                 # the largest score of all lies in the group left out
    assert plain.choose_experts(c, 3, 3, 1)[0][:2] == [2, 3]
    assert plain.choose_experts(c, 3, 1, 1)[0] == [4, 1, 2]
    assert plain.choose_experts(c - 2, 4, 3, 2)[0] == [1, 2, 3, 0]          # negative scores stay ahead of what is left out
    assert plain.choose_experts(torch.tensor([0.3, 0.2, 0.9]).double(), 1, 3, 2)[0] == [2]      # groups of one
    u, w = torch.randn(9, 4, generator=g).double(), torch.randn(4, 3, generator=g).double()
    y = plain.causal_conv(u, w)
    for t in range(9):
        assert torch.allclose(y[t], sum(w[:, j] * u[t - 2 + j] for j in range(3) if t - 2 + j >= 0))


def test_every_mechanism_of_the_plain_model_moves_its_logits():
    w = {k: v.double() for k, v in plain.random_weights(CFG, 1).items()}
    toks = torch.randint(0, 70, (45,), generator=torch.Generator().manual_seed(5)).tolist()
    base = plain.forward(w, CFG, toks)
    top = base.abs().max()

    def moved(cfg=CFG, weights=w):
        return ((plain.forward(weights, cfg, toks) - base).abs().max(-1).values / top).max().item()
    for path, value in [(("layers", 1, "mixer", "mask", "size"), 10), (("layers", 1, "mixer", "mask", "size"), 12), (("layers", 1, "mixer", "rot", "base"), 9.0),
                        (("layers", 1, "mixer", "rot", "scaling", "factor"), 1.5), (("layers", 1, "mixer", "rot", "scaling", "slow"), 3.0),
                        (("layers", 0, "mixer", "gate_cap"), 1.0), (("layers", 0, "mlp", "router", "groups", "keep"), 1), (("logit_scale",), 0.5),
                        (("embedding", "scale"), 1.0), (("layers", 1, "mixer", "scale"), 0.5)]:
        assert moved(changed(path, value)) > 1e-3, path
    for name in plain.tensor_shapes(CFG):
        if ".e" in name and not name.endswith(".e0.gate"):
            continue
        x = dict(w)
        x[name] = x[name] * 0.5 + 0.1
        assert moved(weights=x) > 2e-4, name


def test_the_chunks_of_a_step_cover_every_token_once():
    from ullm_amd.parts.base import StepShape
    from ullm_amd.parts.memory import plan_memory_chunks
    lens = (1, 16, 17, 40, 2)
    p = plan_memory_chunks(StepShape(lens, (0,) * 5))
    items = p.arrays["items"].reshape(-1, 2).tolist()
    assert p.facts == {"num_items": 8} and p.arrays["entry_item"].tolist() == [0, 1, 2, 4, 7]
    at = 0
    for first, n in items:
        assert first == at and 1 <= n <= 16
        at += n
    assert at == sum(lens) and [n for _, n in items] == [1, 16, 16, 1, 16, 16, 8, 2]
    single = plan_memory_chunks(StepShape((1, 1), (5, 9)))
    assert single.facts == {"num_items": 0} and all(a.size == 0 for a in single.arrays.values())
