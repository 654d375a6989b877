"""Nadevik without a GPU: the configuration reader and what it refuses, the plan it becomes (tensor names and shapes, what
a block keeps, latents that another layer reads), cache groups with one row per many tokens, the lists of completed blocks
and of scan segments, and the plain implementation's own pieces against explicit loops."""
import copy
import math
import random

import numpy as np
import pytest
import torch

import plain_nadevik as plain
from ullm_amd.cache.manager import CacheGroupSpec, CacheManager
from ullm_amd.config import ConfigError, NadevikConfig
from ullm_amd.models import build_model
from ullm_amd.parts import KVNeed, StateNeed, StepShape, cache_needs_of
from ullm_amd.parts.pooled import block_planner
from ullm_amd.parts.position import Rotary
from ullm_amd.parts.ssm import plan_scan_segments

MOE = dict(kind="moe", router=dict(experts=6, top=2, groups=dict(count=3, keep=2)), expert=dict(ff=10, limit=2.5))


def parallel(window=9, pool=4, mlp=MOE, **left):
    a = dict(heads=6, kv_heads=2, dim=10, vdim=14, conv=3, scale=0.3, softcap=15.0, mask=dict(size=window, pool=pool))
    a.update(left)
    return dict(type="parallel", mlp=mlp, mixer=dict(left=a, right=dict(inner=20, state=5, dt_rank=3, conv=4), left_scale=0.7, right_scale=1.2))


def latent(window=11, kv_from=None, mlp=MOE, rot_dim=6, **more):
    m = dict(heads=3, dim=8, rot_dim=rot_dim, vdim=12, kv_rank=18, scale=0.25, mask=dict(size=window), rot=dict(base=500.0, dims=rot_dim))
    if kv_from is not None:
        m["kv_from"] = kv_from
    m.update(more)
    return dict(type="latent_attention", mixer=m, mlp=mlp)


CFG = dict(architecture="Nadevik", vocab=70, width=24, norm=dict(eps=1e-4), canon=dict(taps=4),
           embedding=dict(scale=2.0, bigram=dict(buckets=11, mul_prev=5, mul_cur=3)),
           layers=[parallel(), latent(), latent(window=30, kv_from=1), parallel(mlp=None)])


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
    assert isinstance(cfg, NadevikConfig) and cfg.num_hidden_layers == 4 and cfg.canon_taps == 4
    declared = {d.name: tuple(d.shape) for d in model.weight_decls() if d.alias_of is None}
    assert declared == plain.tensor_shapes(CFG)
    assert [(d.name, d.alias_of) for d in model.weight_decls() if d.alias_of is not None] == [("head", "embed")]
    # without a bigram there is no such table, and none of its state
    c = copy.deepcopy(CFG)
    del c["embedding"]["bigram"]
    _, model = build_model(c)
    assert {d.name for d in model.weight_decls() if d.alias_of is None} == set(plain.tensor_shapes(c)) and model.embedder.cache_need() is None


def test_what_the_layers_keep():
    _, model = build_model(CFG)
    groups, _, states = model.cache_layout()
    by = {(g.num_kv_heads, g.tokens_per_row): g for g in groups}
    # windowed tokens and pooled rows of the two parallel layers; one group of latents, as far back as its widest reader looks
    assert len(groups) == 3
    assert by[(2, 1)].window == 9 and len(by[(2, 1)].layers) == 2 and by[(2, 1)].head_dim == 32
    assert by[(2, 4)].window == 0 and len(by[(2, 4)].layers) == 2
    assert by[(1, 1)].window == 30 and by[(1, 1)].layers == ((1, 1),)
    assert model.borrowed_caches() == {(2, 1): (1, 1)}
    conv, inner = 2 * (6 + 2 * 2) * 32, 3 * 20 + 20 * 5
    assert sorted(n.shape[0] for n in states.values()) == sorted([1] + 4 * [3 * 24] + 2 * [conv, inner])
    assert all(n.graph_safe for n in states.values())
    needs = cache_needs_of(model.blocks[0])
    assert [type(n) for n in needs] == [StateNeed, KVNeed, KVNeed, StateNeed, StateNeed]


def test_a_window_shorter_than_a_block_keeps_the_block_s_tokens():
    c = changed(("layers", 0, "mixer", "left", "mask"), dict(size=3, pool=13))
    _, model = build_model(c)
    kv = [n for n in cache_needs_of(model.blocks[0]) if isinstance(n, KVNeed)]
    assert [(n.window, n.tokens_per_row) for n in kv] == [(13, 1), (0, 13)]


@pytest.mark.parametrize("path,value", [
    (("layers",), []), (("layers", 0, "type"), "gla"), (("layers", 0, "mixer", "left"), None), (("layers", 0, "mixer", "right"), None),
    (("layers", 0, "mixer", "left", "kv_heads"), 4), (("layers", 0, "mixer", "left", "mask"), dict(pool=4)),
    (("layers", 0, "mixer", "right", "dt_rank"), 0), (("layers", 1, "mixer", "rot_dim"), 5), (("layers", 1, "mixer", "rot", "dims"), 4),
    (("layers", 2, "mixer", "kv_from"), 0), (("layers", 2, "mixer", "kv_from"), 2), (("layers", 2, "mixer", "kv_from"), 3),
    (("layers", 2, "mixer", "kv_rank"), 20), (("layers", 2, "mixer", "rot", "base"), 7.0), (("layers", 1, "mixer", "kv_from"), 2),
    (("layers", 0, "mlp", "kind"), "dense"), (("layers", 0, "mlp", "router", "groups", "count"), 4),
    (("layers", 0, "mlp", "router", "groups", "keep"), 4), (("layers", 0, "mlp", "router", "top"), 5),
    (("layers", 0, "mlp", "expert", "limit"), 0.0), (("canon",), {}), (("vocab",), KeyError), (("norm",), {})])
def test_configurations_that_are_refused(path, value):
    with pytest.raises(ConfigError):
        NadevikConfig.from_dict(changed(path, value))


def test_angles_formed_in_64_bit():
    table = Rotary.make_table(6, 500.0, 5000, exact=True)
    for p in (0, 1, 77, 4999):
        for i in range(3):
            a = p * 500.0 ** (-2.0 * i / 6)
            assert abs(table[p, i].item() - math.cos(a)) < 1e-7 and abs(table[p, 3 + i].item() - math.sin(a)) < 1e-7


# ----------------------------------------------------------------------------- the cache

def test_a_group_with_one_row_per_many_tokens():
    specs = [CacheGroupSpec(2, 32, 9, ((0, 1),)), CacheGroupSpec(2, 32, 0, ((0, 2),), None, 5)]
    assert [s.rows_for(14) for s in specs] == [14, 2] and [s.pages_beside(20, 3) for s in specs] == [20, 7]
    assert specs[1].bytes_per_token(2) == -(-2 * 2 * 32 * 2 // 5)
    c = CacheManager(specs, [20, 7], 4, 3)
    assert c.pages_for(19) == [5, 1] and c.pages_for(20) == [5, 1] and c.pages_for(24) == [6, 1] and c.pages_for(25) == [7, 2]
    a = c.admit("a")
    assert c.reserve(a, 4)
    assert [len(t) for t in a.tables] == [1, 0]             # no block is complete yet: no page
    c.commit(a, 4)
    assert c.reserve(a, 1) and [len(t) for t in a.tables] == [2, 1]
    c.commit(a, 1)
    c.check()
    for _ in range(70):                                       # one by one; the windowed group gives pages back, the other keeps all
        assert c.reserve(a, 1)
        c.commit(a, 1)
    c.check()
    assert len(a.pages_held(1)) == -(-(75 // 5) // 4) and len(a.pages_held(0)) <= 4
    c.release(a)
    assert c.num_free_pages(0) == 20 and c.num_free_pages(1) == 7


def test_many_requests_never_lack_rows_where_they_have_tokens():
    rng = random.Random(3)
    for pool in (2, 3, 7, 40):
        specs = [CacheGroupSpec(1, 32, 0, ((0, 0),)), CacheGroupSpec(1, 32, 0, ((0, 1),), None, pool)]
        c = CacheManager(specs, [s.pages_beside(24, 4) for s in specs], 4, 4)
        live = {}
        for step in range(300):
            if len(live) < 4 and rng.random() < 0.4:
                live[step] = c.admit(str(step))
            for k in list(live):
                n = rng.choice([1, 1, 2, 9])
                if c.pages_needed(live[k], n)[0] <= c.num_free_pages(0):
                    assert c.reserve(live[k], n)
                    c.commit(live[k], n)
                elif rng.random() < 0.5:
                    c.release(live.pop(k))
            c.check()


@pytest.mark.parametrize("pool", [1, 2, 5, 16])
def test_every_block_is_listed_in_the_step_that_completes_it(pool):
    rng = random.Random(pool)
    plan = block_planner(pool)
    assert plan is block_planner(pool)
    lens, seen = [0, 0, 0], [[], [], []]
    for _ in range(40):
        n = [rng.choice([1, 1, 2, 3, 17]) for _ in lens]
        if all(x == 1 for x in n):
            n[0] = 2
        p = plan(StepShape(tuple(n), tuple(lens)))
        pairs = p.arrays["blocks"].reshape(-1, 2).tolist()
        assert p.facts["num_blocks"] == len(pairs)
        for b, block in pairs:
            assert lens[b] < (block + 1) * pool <= lens[b] + n[b]
            seen[b].append(block)
        lens = [a + b for a, b in zip(lens, n)]
    for total, blocks in zip(lens, seen):
        assert blocks == list(range(total // pool))
    single = plan(StepShape((1, 1), (pool - 1, 0)))
    assert single.facts["num_blocks"] == 0 and single.arrays["blocks"].size == 0


def test_the_segments_of_a_scan_cover_every_token_once():
    lens = (1, 64, 65, 200, 7)
    p = plan_scan_segments(StepShape(lens, (0,) * 5))
    items = p.arrays["items"].reshape(-1, 4).tolist()
    chains = p.arrays["chains"].reshape(-1, 3).tolist()
    assert p.facts == {"num_items": 9, "num_chains": 2} and chains == [[2, 2, 2], [3, 4, 4]]
    at = 0
    for b, first, n, what in items:
        assert first == at and 1 <= n <= 64
        at += n
    assert at == sum(lens)
    assert [i[3] for i in items] == [0, 0, 1, 2, 1, 1, 1, 2, 0]
    assert plan_scan_segments(StepShape((1, 1), (5, 9))).facts == {"num_items": 0, "num_chains": 0}


# ----------------------------------------------------------------------------- the plain implementation itself

def test_plain_convolution_masks_blocks_and_choice_against_loops():
    g = torch.Generator().manual_seed(1)
    u, w = torch.randn(9, 4, generator=g).double(), torch.randn(4, 3, generator=g).double()
    y = plain.causal_conv(u, w)
    for t in range(9):
        want = sum(w[:, j] * u[t - 2 + j] for j in range(3) if t - 2 + j >= 0)
        assert torch.allclose(y[t], want)
    T, window, pool = 40, 7, 5
    tok, blk = plain.seen_tokens(T, window), plain.seen_blocks(T, window, pool)
    for i in range(T):
        assert torch.nonzero(tok[i]).flatten().tolist() == list(range(max(0, i - 6), i + 1))
        assert torch.nonzero(blk[i]).flatten().tolist() == [b for b in range(T // pool) if b * pool + pool - 1 <= i - window]
    # the tokens between the last visible block and the window are seen by nothing
    i = 23
    covered = {b * pool + k for b in torch.nonzero(blk[i]).flatten().tolist() for k in range(pool)} | set(torch.nonzero(tok[i]).flatten().tolist())
    assert set(range(i + 1)) - covered == {15, 16}
    x = torch.randn(13, 2, 3, generator=g).double()
    assert torch.allclose(plain.block_means(x, 4)[2], x[8:12].mean(0)) and plain.block_means(x, 4).shape[0] == 3
    s = torch.tensor([0.1, 0.5, 0.3, 0.3, 0.05, 0.35]).double()
    assert plain.choose_experts(s, 3, 3, 2)[0] == [1, 5, 0]         # groups (0 1), (2 3), (4 5): the middle one is left out
    assert plain.choose_experts(s, 3, 1, 1)[0] == [1, 5, 2]
    assert plain.bigram_rows([3, 4, 9], 11, 5, 3) == [11, (3 * 5 + 4 * 3) % 11, (4 * 5 + 9 * 3) % 11]


def test_plain_scan_and_rotation_against_loops():
    g = torch.Generator().manual_seed(2)
    T, c, n = 6, 3, 2
    x, dt = torch.randn(T, c, generator=g).double(), torch.rand(T, c, generator=g).double()
    A, B, C, D = -torch.rand(c, n, generator=g).double(), torch.randn(T, n, generator=g).double(), torch.randn(T, n, generator=g).double(), torch.randn(c, generator=g).double()
    y = plain.selective_scan(x, dt, A, B, C, D)
    for ch in range(c):
        S = [0.0] * n
        for t in range(T):
            out = D[ch].item() * x[t, ch].item()
            for k in range(n):
                S[k] = math.exp(dt[t, ch].item() * A[ch, k].item()) * S[k] + dt[t, ch].item() * x[t, ch].item() * B[t, k].item()
                out += S[k] * C[t, k].item()
            assert abs(y[t, ch].item() - out) < 1e-12
    v = torch.randn(5, 1, 6, generator=g).double()
    r = plain.rotate_adjacent(v, torch.arange(5), 4, 100.0)
    for p in range(5):
        for i in range(2):
            a = p * 100.0 ** (-2.0 * i / 4)
            assert abs(r[p, 0, 2 * i].item() - (v[p, 0, 2 * i] * math.cos(a) - v[p, 0, 2 * i + 1] * math.sin(a)).item()) < 1e-12
            assert abs(r[p, 0, 2 * i + 1].item() - (v[p, 0, 2 * i + 1] * math.cos(a) + v[p, 0, 2 * i] * math.sin(a)).item()) < 1e-12
    assert torch.equal(r[..., 4:], v[..., 4:])


def test_every_mechanism_of_the_plain_model_moves_its_logits():
    w = {k: v.double() for k, v in plain.random_weights(CFG, 1).items()}
    toks = torch.randint(0, 70, (45,), generator=torch.Generator().manual_seed(5)).tolist()
    base = plain.forward(w, CFG, toks)
    top = base.abs().max()

    def moved(cfg=CFG, weights=w):
        return ((plain.forward(weights, cfg, toks) - base).abs().max(-1).values / top).max().item()
    for path, value in [(("layers", 0, "mixer", "left", "mask", "size"), 10), (("layers", 0, "mixer", "left", "mask", "pool"), 5),
                        (("layers", 0, "mixer", "left", "softcap"), 1.0), (("layers", 0, "mixer", "left_scale"), 0.2),
                        (("layers", 1, "mixer", "mask", "size"), 9), (("layers", 2, "mixer", "mask", "size"), 11),
                        (("layers", 1, "mixer", "rot", "base"), 3.0), (("layers", 0, "mlp", "router", "groups", "keep"), 1),
                        (("layers", 0, "mlp", "expert", "limit"), 0.3), (("embedding", "scale"), 1.0), (("embedding", "bigram", "mul_cur"), 4)]:
        assert moved(changed(path, value)) > 1e-3, path
    for name in ("l1.canon1", "l0.mix.left.q.conv", "l0.mix.left.pb", "l0.mix.right.conv", "l0.mix.right.D", "l0.mix.right.A_log",
                 "l0.mix.right.dt.b", "l1.mix.dkv", "l2.mix.g", "l0.norm1", "l1.norm2", "l0.mix.left.k.norm", "bigram"):
        x = dict(w)
        x[name] = x[name] * 0.5 + 0.1
        assert moved(weights=x) > 1e-3, name
