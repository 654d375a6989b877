"""Nadevik in the framework against the plain implementation (``plain_nadevik``, 64-bit): each mechanism's kernels alone
and as one-layer models; the stream after every layer; whole prompts; a prompt and then token by token, also from the
very first token; portions down to two tokens; unequal requests in one batch, in a pool and slots that are used again; long
decoding while windows pass and pages return; scores scaled so that single keys just inside a window, or a block that has
just come into sight, decide a row; state that carries a token hundreds of steps; sizes that differ wherever they can,
also values that make things equal or one; many requests in one captured step; greedy generation through the entry point.
In 32-bit to rounding; in bfloat16, where a rounded router input may choose another expert at a close call, the rows
ahead of the first close call to rounding and the others within a bound that a lost key or a wrong state exceeds."""
import copy
import json
import math
import os
from types import SimpleNamespace

import numpy as np
import pytest
import torch
from safetensors.torch import save_file

import plain_nadevik as plain
from gpu_util import DEV, paged_cache, table_tensor

pytestmark = pytest.mark.gpu

REL = {"float32": 3e-5, "bfloat16": 3e-2}
CLOSE_CALL = 0.05
# bfloat16 bounds (median, 85th of 100 rows, largest row ahead of the first close call)
BF16_BOUNDS = {"B": (4e-2, 1e-1, 0.5)}


def moe(experts, top, ff, limit=2.0, groups=None):
    r = dict(experts=experts, top=top)
    if groups:
        r["groups"] = dict(count=groups[0], keep=groups[1])
    return dict(kind="moe", router=r, expert=dict(ff=ff, limit=limit))


def par(heads, kv, dim, vdim, scale, window, pool=0, conv=3, softcap=15.0, right=(24, 8, 5, 4), scales=(0.8, 1.1), mlp=None):
    left = dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, conv=conv, scale=scale, softcap=softcap)
    if window:
        left["mask"] = dict(size=window, pool=pool)
    return dict(type="parallel", mlp=mlp, mixer=dict(left=left, right=dict(inner=right[0], state=right[1], dt_rank=right[2], conv=right[3]),
                                                     left_scale=scales[0], right_scale=scales[1]))


def lat(heads, dim, rot_dim, vdim, kv_rank, window, kv_from=None, scale=None, base=1000.0, mlp=None):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, scale=scale or (dim + rot_dim) ** -0.5,
             mask=dict(size=window), rot=dict(base=base, dims=rot_dim))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type="latent_attention", mixer=m, mlp=mlp)


def config(width, vocab, layers, taps=3, eps=1e-5, scale=1.0, bigram=(17, 5, 3)):
    e = dict(scale=scale)
    if bigram:
        e["bigram"] = dict(buckets=bigram[0], mul_prev=bigram[1], mul_cur=bigram[2])
    return dict(architecture="Nadevik", vocab=vocab, width=width, norm=dict(eps=eps), canon=dict(taps=taps), embedding=e, layers=layers)


# A: every kind of layer; a reader that looks further back than the layer whose latents it reads, and one that looks less far
CFG_A = config(48, 131, [par(6, 2, 16, 24, 0.3, 21, 6, conv=4, mlp=moe(8, 3, 20, 1.5, (4, 2))), lat(3, 16, 8, 12, 24, 19, mlp=moe(6, 2, 12, 3.0, (2, 1))),
                         lat(5, 8, 8, 20, 24, 33, kv_from=1, mlp=None), lat(2, 24, 8, 8, 24, 7, kv_from=1, mlp=moe(5, 3, 16)),
                         par(4, 4, 24, 8, 0.2, 13, 9, conv=2, right=(40, 16, 3, 3), mlp=moe(9, 2, 8, 0.7, (3, 3)))], taps=4, scale=3.0)
# B: values that make things equal or one, and sizes that no 16-byte access fits: one head, one expert, all experts, one group,
# taps of one, blocks of one token, a window of one, a block longer than the window, no soft cap, no bigram, no rotated dims,
# no window at all, a rank and a state of one
CFG_B = config(40, 97, [par(3, 3, 6, 10, 0.5, 5, 8, conv=1, softcap=0.0, right=(13, 1, 1, 1), scales=(1.0, 1.0), mlp=moe(4, 4, 9, 1.0, (1, 1))),
                        lat(1, 6, 0, 10, 10, 1, mlp=moe(1, 1, 14)), par(1, 1, 10, 6, 0.4, 1, 1, conv=5, right=(9, 6, 2, 6), mlp=None),
                        lat(3, 10, 2, 6, 12, 0, mlp=moe(6, 2, 7, 5.0, (6, 2))), par(4, 1, 16, 16, 0.25, 0, 0, conv=2, right=(16, 3, 8, 2), mlp=moe(3, 1, 33))],
               taps=1, bigram=None)
# C: head sizes of 64 and 128 (and values narrower), 96 and 256 cached dims, states of 64 and 80 (past what a lane holds),
# a window shorter than a page, blocks of 32 tokens
CFG_C = config(64, 211, [par(4, 2, 128, 64, 0.09, 5, 3, conv=4, right=(64, 64, 12, 4), mlp=moe(16, 4, 16, 1.2, (4, 3))), lat(4, 64, 32, 64, 200, 40, mlp=moe(8, 2, 24)),
                         par(8, 2, 64, 64, 0.12, 40, 32, conv=4, softcap=8.0, right=(32, 80, 4, 4), mlp=None)], taps=2, eps=1e-6)
# W: scores of many units under an offset far below zero: a row's weight lies on one or two keys or blocks
CFG_W = config(32, 64, [par(2, 1, 16, 16, 3.0, 33, 5, conv=2, softcap=14.0, right=(8, 4, 2, 2), scales=(1.0, 0.05), mlp=None)], taps=2, scale=1.0)
# L: the same for the latents' window, read by a layer with a wider one
CFG_L = config(32, 64, [lat(2, 16, 4, 16, 16, 17, scale=1.5, mlp=None), lat(2, 16, 4, 16, 16, 41, kv_from=0, scale=1.5, mlp=None)], taps=2)
CFG_PAR = config(32, 64, [par(4, 2, 8, 8, 0.35, 12, 4, mlp=None)], taps=2)
CFG_LAT = config(32, 64, [lat(2, 8, 4, 8, 16, 14, mlp=None)], taps=2)
CFG_MOE = config(32, 64, [lat(1, 8, 4, 8, 8, 10, mlp=moe(12, 3, 8, 1.0, (4, 2)))], taps=3)
CFG_M = config(32, 50, [par(4, 2, 32, 32, 0.2, 6, 2, conv=4, right=(64, 16, 4, 4), mlp=moe(8, 2, 16, 1.0, (4, 2))), lat(2, 16, 16, 16, 16, 5, mlp=None)], taps=3)

MODELS = {"A": (CFG_A, 1), "B": (CFG_B, 2), "C": (CFG_C, 3), "W": (CFG_W, 4), "L": (CFG_L, 5), "M": (CFG_M, 6), "par": (CFG_PAR, 7),
          "lat": (CFG_LAT, 8), "moe": (CFG_MOE, 9)}


def made_weights(name):
    cfg, seed = MODELS[name]
    w = plain.random_weights(cfg, seed)
    if name == "W":
        w["l0.mix.left.pb"] = torch.full_like(w["l0.mix.left.pb"], -9.0)
    if name == "L":
        for t in ("l0.mix.q", "l0.mix.uk", "l1.mix.q", "l1.mix.uk"):
            w[t] = (w[t].float() * 2.5).to(torch.bfloat16)
    return w


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """{name: (folder, config, 64-bit weights)}; the folders hold bfloat16 tensors under the design's names."""
    out = {}
    for name, (cfg, _) in MODELS.items():
        d = tmp_path_factory.mktemp(f"nadevik{name}")
        w = made_weights(name)
        with open(os.path.join(d, "config.json"), "w") as f:
            json.dump(cfg, f)
        save_file({k: v.contiguous() for k, v in w.items()}, os.path.join(d, "model.safetensors"))
        out[name] = (str(d), cfg, {k: v.double() for k, v in w.items()})
    return out


_oracle_cache = {}


def oracle_and_gaps(models, name, toks):
    """(logits [T, vocab], for every row the smallest gap between what was taken and what was left over all routed layers)."""
    key = (name, tuple(toks))
    if key not in _oracle_cache:
        _, cfg, w = models[name]
        plain.MARGINS = []
        logits = plain.forward(w, cfg, list(toks)).float().numpy()
        gaps = np.min([m.numpy() for m in plain.MARGINS], axis=0) if plain.MARGINS else np.full(len(toks), np.inf)
        plain.MARGINS = None
        _oracle_cache[key] = (logits, gaps)
    return _oracle_cache[key]


def close(got, want, dtype, gaps=None, name=""):
    err = np.abs(got - want).max(-1) / float(np.abs(want).max())
    if dtype == "float32":
        assert err.max() <= REL[dtype], f"max {err.max():.3e} at row {int(err.argmax())}"
        return
    assert np.isfinite(got).all()
    mid, most, top = BF16_BOUNDS.get(name, (2.5e-2, 6e-2, 0.3))
    calls = np.nonzero(gaps < CLOSE_CALL)[0] if gaps is not None else []
    sharp = err[:int(calls[0])] if len(calls) else err
    if len(sharp) >= 8:
        assert np.median(sharp) <= mid and np.quantile(sharp, 0.85) <= most, \
            f"median {np.median(sharp):.3e}, 85th {np.quantile(sharp, 0.85):.3e} over {len(sharp)} rows"
    assert not len(sharp) or sharp.max() <= top, f"max {sharp.max():.3e} at row {int(sharp.argmax())}"
    if len(err) >= 8:
        assert np.median(err) <= 0.2, f"median {np.median(err):.3e} behind a close call"


def agree(models, name, toks, got, dtype, rows=None):
    want, gaps = oracle_and_gaps(models, name, toks)
    if rows is not None:
        want, gaps = want[rows], gaps[rows]
    close(got, want, dtype, gaps, name)


def tokens(vocab, n, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


@pytest.fixture(scope="module")
def replayers(models):
    from ullm_amd.replay import Replayer
    made = {}

    def get(name, dtype, max_tokens=512, max_requests=4, use_graphs=True):
        key = (name, dtype, max_tokens, max_requests, use_graphs)
        if key not in made:
            made[key] = Replayer(models[name][0], dtype, max_tokens, 16, DEV, max_requests=max_requests, use_graphs=use_graphs)
        rep = made[key]
        cache = rep.runner.cache
        assert not rep.live and all(cache.num_free_pages(g) == a.num_pages for g, a in enumerate(cache.allocators))
        return rep
    return get


def run(rep, rid, toks, cuts, end=True):
    """Feed ``toks`` in portions of the sizes ``cuts`` (the rest one by one); logits of every position."""
    got, at, step = [], 0, 0
    sizes = list(cuts) + [1] * len(toks)
    while at < len(toks):
        n = min(sizes[step], len(toks) - at)
        got.append(rep.step({"step": step, "entries": [{"id": rid, "tokens": toks[at:at + n], "want": list(range(n))}],
                             "end": [rid] if end and at + n == len(toks) else []}))
        at, step = at + n, step + 1
    return np.concatenate(got)


BIG = [(n, d) for n in ("A", "B", "C") for d in ("float32", "bfloat16")]
ALONE = [(n, d) for n in ("par", "lat", "moe") for d in ("float32", "bfloat16")]


@pytest.mark.parametrize("name,dtype", BIG + ALONE)
def test_whole_prompts(replayers, models, name, dtype):
    rep = replayers(name, dtype)
    for i, n in enumerate((1, 2, 15, 16, 17, 90)):
        toks = tokens(models[name][1]["vocab"], n, 10 + i)
        agree(models, name, toks, run(rep, "r", toks, [n]), dtype)


@pytest.mark.parametrize("name,dtype", [("par", "float32"), ("par", "bfloat16"), ("C", "float32"), ("A", "float32")])
def test_long_portions_of_two_requests_in_one_step(replayers, models, name, dtype):
    """Steps of more than 512 tokens (kernels that take several tokens a block), the second request's tokens off every
    block's edge, then the rest of both."""
    rep = replayers(name, dtype, max_tokens=1280)
    vocab = models[name][1]["vocab"]
    a, b = tokens(vocab, 597, 80), tokens(vocab, 390, 81)
    got = {"a": [], "b": []}
    for step, cut in enumerate(({"a": 333, "b": 279}, {"a": 264, "b": 111})):
        at = {"a": 0 if step == 0 else 333, "b": 0 if step == 0 else 279}
        entries = [{"id": k, "tokens": t[at[k]:at[k] + cut[k]], "want": list(range(cut[k]))} for k, t in (("a", a), ("b", b))]
        out = rep.step({"step": step, "entries": entries, "end": [] if step == 0 else ["a", "b"]})
        got["a"].append(out[:cut["a"]])
        got["b"].append(out[cut["a"]:])
    agree(models, name, a, np.concatenate(got["a"]), dtype)
    agree(models, name, b, np.concatenate(got["b"]), dtype)
    one = run(rep, "r", a, [597])                        # and one request alone, from a page's first row on
    agree(models, name, a, one, dtype)


@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_the_stream_after_every_layer(models, name):
    """Layer by layer in 32-bit: the stream once what the layer left pending is normed and added."""
    from ullm_amd.engine.loading import load_model
    from ullm_amd.engine.runner import ModelRunner, StepEntry
    d, cfg, w = models[name]
    toks = tokens(cfg["vocab"], 50, 3)
    want = []
    plain.forward(w, cfg, toks, want)
    _, model, env = load_model(d, "float32", DEV, context_len=64)
    runner = ModelRunner(model, env, page_size=16, num_pages=4, max_requests=1, use_graphs=False)
    rc = runner.cache.admit("r")
    assert runner.cache.reserve(rc, len(toks))
    ctx, _ = runner.build_context([StepEntry(rc, toks, [])])
    stream = model.embedder.forward(ctx, runner.caches.get(-1))
    pending = None
    for i, (block, cache_id) in enumerate(model.run_order):
        cache = runner.caches.get(cache_id)
        stream, pending = model.blocks[block].forward(stream, pending, ctx, cache)
        y = pending.joined().double()
        after = (stream.double() + plain.rms_norm(y, pending.post.gain.double(), pending.post.eps)).cpu()
        assert (after - want[i]).abs().max() <= 3e-5 * want[i].abs().max(), i


@pytest.mark.parametrize("name,dtype", BIG)
def test_a_prompt_and_then_token_by_token(replayers, models, name, dtype):
    toks = tokens(models[name][1]["vocab"], 90, 15)
    for graphs in (True, False):
        agree(models, name, toks, run(replayers(name, dtype, use_graphs=graphs), "r", toks, [40]), dtype)


@pytest.mark.parametrize("name,dtype", BIG)
def test_token_by_token_from_the_first_token(replayers, models, name, dtype):
    toks = tokens(models[name][1]["vocab"], 50, 16)
    agree(models, name, toks, run(replayers(name, dtype), "r", toks, []), dtype)


@pytest.mark.parametrize("name,dtype", BIG)
@pytest.mark.parametrize("cuts", [(2, 2, 3, 2, 14, 2, 17, 31, 2), (1, 1, 2, 30, 3, 3, 33), (16, 16, 16, 2, 25), (2,) * 45])
def test_portions_of_changing_size(replayers, models, name, dtype, cuts):
    toks = tokens(models[name][1]["vocab"], 90, 15)
    got = run(replayers(name, dtype), "r", toks, cuts)
    agree(models, name, toks, got, dtype)


@pytest.mark.parametrize("name,dtype", BIG)
def test_unequal_requests_together_in_pages_and_slots_used_again(replayers, models, name, dtype):
    """Six requests through two slots and a pool of 128 tokens: portions beside single tokens, a request left out of a
    step, a request that starts in the slot and pages another has just given back."""
    rep = replayers(name, dtype, max_tokens=128, max_requests=2)
    vocab = models[name][1]["vocab"]
    reqs = {f"q{i}": tokens(vocab, n, 30 + i) for i, n in enumerate((50, 33, 1, 64, 20, 47))}
    plan = [[("q0", 20), ("q1", 2)], [("q0", 1), ("q1", 31)], [("q0", 29)],          # q1 ends; q0 goes on alone
            [("q2", 1)], [("q3", 17)], [("q3", 1)], [("q3", 2)], [("q3", 44)],        # q2 and q3 use q1's and q0's slots again
            [("q4", 3), ("q5", 30)], [("q5", 1)], [("q4", 16), ("q5", 1)], [("q4", 1), ("q5", 15)]]
    at, got = {r: 0 for r in reqs}, {r: [] for r in reqs}
    for s, entries in enumerate(plan):
        msg = {"step": s, "entries": [], "end": []}
        for r, n in entries:
            msg["entries"].append({"id": r, "tokens": reqs[r][at[r]:at[r] + n], "want": list(range(n))})
            at[r] += n
            if at[r] == len(reqs[r]):
                msg["end"].append(r)
        out, row = rep.step(msg), 0
        for r, n in entries:
            got[r].append(out[row:row + n])
            row += n
    assert at == {r: len(t) for r, t in reqs.items()}
    for r, toks in reqs.items():
        agree(models, name, toks, np.concatenate(got[r]), dtype)
    rep.runner.cache.check()


def test_many_single_tokens_in_one_captured_step(replayers, models):
    """140 requests a step, one token each, nine steps (windows and blocks pass): captured steps that are replayed against
    the same steps run eagerly and against the plain implementation."""
    vocab = models["M"][1]["vocab"]
    reqs = {f"m{i}": tokens(vocab, 9, 200 + i) for i in range(140)}
    got = {}
    for graphs in (True, False):
        rep = replayers("M", "bfloat16", max_tokens=140 * 16, max_requests=140, use_graphs=graphs)
        rows = {r: [] for r in reqs}
        for step in range(9):
            out = rep.step({"step": step, "entries": [{"id": r, "tokens": [t[step]], "want": [0]} for r, t in reqs.items()],
                            "end": list(reqs) if step == 8 else []})
            for i, r in enumerate(reqs):
                rows[r].append(out[i])
        got[graphs] = {r: np.stack(v) for r, v in rows.items()}
    for r in list(reqs)[::7]:
        agree(models, "M", reqs[r], got[True][r], "bfloat16")
    diff = max(np.abs(got[True][r] - got[False][r]).max() / np.abs(got[False][r]).max() for r in reqs)
    assert diff <= 1e-2, diff


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_while_windows_pass_and_pages_return(replayers, models, dtype):
    """190 tokens one by one through captured steps: the windows pass many pages, which go back to the pool, blocks come
    into sight one after the other, states carry on; a second request then takes the pages and the slot again."""
    rep = replayers("A", dtype, max_tokens=192)
    toks = tokens(models["A"][1]["vocab"], 190, 40)
    agree(models, "A", toks, run(rep, "r", toks, [3]), dtype)
    other = tokens(models["A"][1]["vocab"], 100, 41)
    agree(models, "A", other, run(rep, "s", other, [60]), dtype)


EDGE_CUTS = [(200,), (120,), (17, 64, 2, 31, 2, 30), (33, 33, 1, 1, 47, 47, 2, 16), (32, 1, 1, 1, 66, 34)]


@pytest.mark.parametrize("name", ["W", "L"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cuts", EDGE_CUTS)
def test_single_keys_and_blocks_decide(replayers, models, name, dtype, cuts):
    """Scores of many units: a row's weight lies on one or two keys or blocks, in portions and for single tokens: a window
    one key too long, a block seen a token early, or a key lost at a page's border moves the row."""
    toks = tokens(models[name][1]["vocab"], 200, 42)
    want, _ = oracle_and_gaps(models, name, toks)
    got = run(replayers(name, dtype), "r", toks, cuts)
    if dtype == "float32":
        close(got, want, dtype)
    else:
        err = np.abs(got - want).max(-1) / np.abs(want).max()
        assert np.median(err) < 4e-2 and err.max() < 0.3, (np.median(err), err.max())


def test_edges_decide_rows_in_the_peaked_models(models):
    """The plain implementation itself: with a window or block one token longer or shorter, or blocks that come into sight a
    token early or late, several rows move by far more than the bounds above."""
    toks = tokens(64, 200, 42)

    def moved(name, change=None, seen=None):
        _, cfg, w = models[name]
        c = copy.deepcopy(cfg)
        if change:
            change(c["layers"])
        base, keep = plain.forward(w, cfg, toks), plain.seen_blocks
        if seen:
            plain.seen_blocks = lambda T, window, pool: keep(T, window + seen, pool)
        try:
            m = (plain.forward(w, c, toks) - base).abs().max(-1).values / base.abs().max()
        finally:
            plain.seen_blocks = keep
        return int((m > 0.03).sum())
    for size in (32, 34):
        assert moved("W", lambda L: L[0]["mixer"]["left"]["mask"].update(size=size)) >= 3, size
    for pool in (4, 6):
        assert moved("W", lambda L: L[0]["mixer"]["left"]["mask"].update(pool=pool)) >= 3, pool
    for seen in (-1, 1):
        assert moved("W", seen=seen) >= 3, seen
    for layer, size in ((0, 16), (0, 18), (1, 40), (1, 42)):
        assert moved("L", lambda L: L[layer]["mixer"]["mask"].update(size=size)) >= 3, (layer, size)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cuts", [(300,), (1, 150, 2, 100), (290,)])
def test_a_token_hundreds_of_steps_back_is_still_there(replayers, models, dtype, cuts):
    """The slowest channels of the scan and the first block still hold the first tokens after 300 steps: the last logits
    move when the first token is another one (in the plain implementation), and the framework follows."""
    _, cfg, _ = models["par"]
    toks = tokens(cfg["vocab"], 300, 44)
    other = [(toks[0] + 1) % cfg["vocab"]] + toks[1:]
    base, changed = oracle_and_gaps(models, "par", toks)[0], oracle_and_gaps(models, "par", other)[0]
    assert np.abs(base[-1] - changed[-1]).max() > 5e-4 * np.abs(base).max()
    got = run(replayers("par", dtype), "r", toks, cuts)
    agree(models, "par", toks, got, dtype)
    if dtype == "float32":
        got_other = run(replayers("par", dtype), "r", other, cuts)
        moved, want_moved = got_other[-1] - got[-1], changed[-1] - base[-1]
        assert np.abs(moved - want_moved).max() <= 0.05 * np.abs(want_moved).max()


@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_greedy_generation_through_the_entry_point(models, name):
    from ullm_amd import LLM, EngineConfig, SamplingParams
    d, cfg, w = models[name]
    g = torch.Generator().manual_seed(50)
    prompts = [torch.randint(0, cfg["vocab"], (n,), generator=g).tolist() for n in (5, 19, 1, 33)]
    expected = [plain.greedy_generate(w, cfg, p, 10) for p in prompts]
    for kw in (dict(), dict(max_num_batched_tokens=12, max_prefill_chunk=5, max_bs=3), dict(enforce_eager=True, disable_async_scheduling=True),
               dict(num_pages=6)):
        args = dict(model=d, dtype="float32", max_bs=8, context_len=128, page_size=16, num_pages=24, device=DEV)
        args.update(kw)
        llm = LLM(EngineConfig(**args))
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=10, ignore_eos=True))
        for e, o in zip(expected, outs):
            assert o.token_ids == e
        cache = llm.engine.runner.cache
        cache.check()
        assert all(cache.num_free_pages(i) == a.num_pages for i, a in enumerate(cache.allocators))
        llm.shutdown()


def test_the_trace_program_runs_the_design(models, trace_run):
    d, cfg, _ = models["A"]
    toks = tokens(cfg["vocab"], 40, 60)
    want, _ = oracle_and_gaps(models, "A", toks)
    tr = trace_run(d, "float32", 128)
    a = tr.step([("a", toks[:21], [0, 20])])
    b = tr.step([("a", toks[21:], [18])], end=["a"])
    tr.close()
    close(np.concatenate((a, b)), want[[0, 20, 39]], "float32")


def test_random_weights_for_the_named_size():
    from ullm_amd.config import parse_random_weights
    from ullm_amd.models import build_model
    config, _ = parse_random_weights("nadevik-2048")
    cfg, model = build_model(config)
    assert cfg.hidden_size == 2048 and len(model.blocks) == 8 and model.borrowed_caches()


# ------------------------------------------------------------------------------------------- kernels alone

def step_context(lens, starts=None, slots=None):
    """What the kernels read of a step with entries of these lengths (slots in another order than the entries)."""
    q = np.concatenate(([0], np.cumsum(lens))).astype(np.int32)
    starts = starts or [0] * len(lens)
    to = lambda a: torch.from_numpy(np.ascontiguousarray(np.asarray(a, dtype=np.int32))).to(DEV)      # noqa: E731
    return SimpleNamespace(q_start=to(q), token_entry=to(np.repeat(np.arange(len(lens)), lens)), num_entries=len(lens),
                           entry_slot=to(slots if slots is not None else np.arange(len(lens))[::-1] + 1),
                           positions=to(np.concatenate([s + np.arange(n) for s, n in zip(starts, lens)])),
                           decode_only=all(n == 1 for n in lens))


STEPS = ([37, 1, 70], [2, 18, 1], [1, 1, 1], [1, 1, 1])
LONG_STEPS = ([301, 2, 1], [1, 1800, 270], [5, 1, 1])


@pytest.mark.parametrize("channels,taps", [(24, 1), (24, 2), (300, 3), (1028, 4), (7, 4), (40, 9)])
@pytest.mark.parametrize("mode", ["silu", "residual"])
@pytest.mark.parametrize("steps", [STEPS, LONG_STEPS], ids=["short", "long"])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_short_convolution_alone(channels, taps, mode, steps, dtype):
    """Three requests in several steps; the inputs in columns of wider rows, the state behind other values."""
    from ullm_amd.kernels import ops
    g = torch.Generator().manual_seed(channels + taps)
    xs = [torch.randn(sum(s[i] for s in steps), channels, generator=g).to(dtype) for i in range(3)]
    w, bias = torch.randn(channels, taps, generator=g), torch.randn(channels, generator=g)
    off = 4
    state = torch.full((5, off + max(1, (taps - 1) * channels)), 3.0, device=DEV)
    state[:, off:] = 0.0
    at, got = [0, 0, 0], [[], [], []]
    for lens in steps:
        ctx = step_context(lens)
        rows = torch.cat([x[a:a + n] for x, a, n in zip(xs, at, lens)])
        wide = torch.cat((torch.randn(rows.shape[0], 8).to(dtype), rows), dim=1).to(DEV)
        out = ops.short_conv(wide[:, 8:], w.t().contiguous().to(DEV), bias.to(DEV) if mode == "silu" else None, state, off, ctx,
                             ops.CONV_SILU if mode == "silu" else ops.CONV_RESIDUAL, dtype)
        row = 0
        for i, n in enumerate(lens):
            got[i].append(out[row:row + n].double().cpu())
            row += n
            at[i] += n
    for x, y in zip(xs, got):
        c = plain.causal_conv(x.double(), w.double())
        want = plain.silu(c + bias.double()) if mode == "silu" else x.double() + c
        assert (torch.cat(y) - want).abs().max() <= (2e-6 if dtype == torch.float32 else 1e-2) * want.abs().max()
    assert bool((state[:, :off] == 3.0).all()) and bool((state[0, off:] == 0).all()) and bool((state[4, off:] == 0).all())
    if taps > 1:
        assert torch.equal(state[3, off:].view(taps - 1, channels).cpu(), xs[0][-(taps - 1):].float())


@pytest.mark.parametrize("inner,N", [(5, 1), (24, 6), (100, 8), (70, 16), (64, 32), (200, 24), (16, 64), (33, 80), (20, 200)])
@pytest.mark.parametrize("segments", [True, False])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_selective_scan_alone(inner, N, segments, dtype):
    """Three requests in four steps (portions of up to 70 tokens: two segments; then single tokens), step sizes from tiny
    to large; in segments side by side, and every entry in order."""
    from ullm_amd.kernels import ops
    from ullm_amd.parts.base import StepShape
    from ullm_amd.parts.ssm import plan_scan_segments
    g = torch.Generator().manual_seed(inner * 100 + N)
    A = -torch.rand(inner, N, generator=g).double() * 6 - 0.001
    D, bias = torch.randn(inner, generator=g), torch.randn(inner, generator=g) - 2
    seqs = []
    for i in range(3):
        n = sum(s[i] for s in STEPS)
        seqs.append((torch.randn(n, inner, generator=g).to(dtype), torch.randn(n, inner, generator=g) * 2, torch.randn(n, 2 * N, generator=g).to(dtype),
                     torch.randn(n, inner, generator=g).to(dtype)))
    want = []
    for x, raw, bc, z in seqs:
        dt = torch.nn.functional.softplus(raw.double() + bias.double(), threshold=1e9)
        want.append(plain.selective_scan(x.double(), dt, A, bc[:, :N].double(), bc[:, N:].double(), D.double()) * plain.silu(z.double()))
    a_log2 = (A * math.log2(math.e)).float().to(DEV)
    off = 8
    state = torch.full((5, off + inner * N), 3.0, device=DEV)
    state[:, off:] = 0.0
    at, got = [0, 0, 0], [[], [], []]
    for lens in STEPS:
        ctx = step_context(lens)
        cat = lambda k: torch.cat([s[k][a:a + n] for s, a, n in zip(seqs, at, lens)]).to(DEV)        # noqa: E731
        wide = torch.cat((cat(0), cat(3)), dim=1)                      # x and z as columns of one row
        plan = plan_scan_segments(StepShape(tuple(lens), (0, 0, 0)))
        plan.arrays = {k: torch.from_numpy(v).to(DEV) for k, v in plan.arrays.items()}
        out = ops.selective_scan(wide[:, :inner], cat(1), cat(2), wide[:, inner:], a_log2, bias.to(DEV), D.to(DEV), state, off, ctx,
                                 plan if segments else None)
        row = 0
        for i, n in enumerate(lens):
            got[i].append(out[row:row + n].double().cpu())
            row += n
            at[i] += n
    for w, y in zip(want, got):
        assert (torch.cat(y) - w).abs().max() <= (2e-5 if dtype == torch.float32 else 1e-2) * w.abs().max()
    assert bool((state[:, :off] == 3.0).all()) and bool((state[0, off:] == 0).all()) and bool((state[4, off:] == 0).all())


@pytest.mark.parametrize("nq,nkv,hd", [(3, 3, 32), (8, 2, 64), (6, 1, 96), (4, 2, 128), (2, 2, 256), (40, 2, 32), (4, 2, 48), (5, 5, 10)])
@pytest.mark.parametrize("window,pool", [(0, 0), (1, 1), (21, 0), (37, 5), (64, 16), (5, 40)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_attention_over_a_window_and_blocks_alone(nq, nkv, hd, window, pool, dtype):
    """Decoded tokens beside portions, at positions around the windows' and blocks' edges; unused rows of the pools hold
    NaN.  With and without a soft cap; decode launches of several splits and waves; the softmax through the general kernel."""
    from ullm_amd.kernels import ops
    from ullm_amd.parts.attention import plan_attention_step
    from ullm_amd.parts.base import StepShape
    g = torch.Generator().manual_seed(nq * 1000 + hd + window)
    totals, lens = [150, 38, 97, 1, 70], [1, 1, 60, 1, 35]
    starts = [t - n for t, n in zip(totals, lens)]
    P = 16
    ks = [torch.randn(t, nkv, hd, generator=g).to(dtype) for t in totals]
    vs = [torch.randn(t, nkv, hd, generator=g).to(dtype) for t in totals]
    k_pool, v_pool, tables = paged_cache(ks, vs, P, dtype, DEV, seed=1)
    ctx = step_context(lens, starts)
    group = SimpleNamespace(block_table=table_tensor(tables, DEV), page_size=P)
    pooled = dict()
    if pool:
        mk = [plain.block_means(k.double(), pool).to(dtype) for k in ks]
        mv = [plain.block_means(v.double(), pool).to(dtype) for v in vs]
        pk, pv, ptab = paged_cache(mk, mv, P, dtype, DEV, seed=2)
        pooled = dict(pool=pool, pooled_group=SimpleNamespace(block_table=table_tensor(ptab, DEV, max(1, max(len(t) for t in ptab))), page_size=P), pk_pool=pk, pv_pool=pv)
    q = torch.randn(sum(lens), nq, hd, generator=g).to(dtype)
    bias = torch.randn(nq, generator=g) - 1
    scale = 2.0 * hd ** -0.5
    plan = plan_attention_step(StepShape(tuple(lens), tuple(starts)))
    plan.arrays = {k: torch.from_numpy(v).to(DEV) for k, v in plan.arrays.items()}

    def expected(cap, softmax):
        out, row = [], 0
        for i, n in enumerate(lens):
            T = totals[i]
            seen = plain.seen_tokens(T, window)[starts[i]:]
            keys, values = ks[i].double(), vs[i].double()
            if pool:
                keys, values = torch.cat((keys, mk[i].double())), torch.cat((values, mv[i].double()))
                seen = torch.cat((seen, plain.seen_blocks(T, window, pool)[starts[i]:]), dim=1)
            o = torch.zeros(n, nq, hd, dtype=torch.float64)
            for h in range(nq):
                kv = h // (nq // nkv)
                s = plain.capped((q[row:row + n, h].double() @ keys[:, kv].T) * scale, cap) + bias[h].double()
                w = torch.softmax(s.masked_fill(~seen, -math.inf), -1) if softmax else torch.sigmoid(s) * seen
                o[:, h] = w @ values[:, kv]
            out.append(o)
            row += n
        return torch.cat(out).reshape(sum(lens), nq * hd)
    for cap, softmax, split in ((3.0, False, {}), (0.0, False, {}), (3.0, False, dict(splits=3, waves=1)), (3.0, False, dict(splits=2, waves=4)),
                                (3.0, True, {})):
        got = ops.pooled_attention(q.reshape(sum(lens), nq * hd).to(DEV), k_pool, v_pool, ctx, group, nq, nkv, hd, scale, window, plan, cap,
                                   bias.to(DEV), softmax=softmax, **split, **pooled).double().cpu()
        want = expected(cap, softmax)
        assert torch.isfinite(got).all()
        err = (got - want).abs().max() / want.abs().max()
        assert err <= (2e-5 if dtype == torch.float32 else 1.5e-2), (cap, softmax, split, float(err))


@pytest.mark.parametrize("H", [8, 40, 300, 2048, 33])
@pytest.mark.parametrize("second", [None, "plain", "stack"])
def test_what_lies_between_two_sublayers(H, second):
    """A branch, two weighted branches, stacks of partial sums; the new rows out in either dtype or not at all; with the
    convolution over the rows in the state."""
    from ullm_amd.kernels import ops
    g = torch.Generator().manual_seed(H)
    T, eps, a, b = 9, 1e-5, 0.7, -1.3
    x, gain = torch.randn(T, H, generator=g), 1 + 0.2 * torch.randn(H, generator=g)
    ya, yb = torch.randn(3, T, H, generator=g), torch.randn(2, T, H, generator=g)
    for dtype in (torch.float32, torch.bfloat16):
        first = ya[0].to(dtype)
        y = a * first.double()
        if second == "plain":
            other = yb[0].to(dtype)
            y = y + b * other.double()
        elif second == "stack":
            first, other = ya, yb
            y = a * ya.double().sum(0) + b * yb.double().sum(0)
        else:
            other = None
        new = x.double() + plain.rms_norm(y, gain.double(), eps)
        kw = dict(second=None if other is None else other.to(DEV), a=a, b=b)
        for out_dtype in (None, torch.float32, torch.bfloat16):
            s = x.clone().to(DEV)
            got = ops.post_add(first.to(DEV), s, gain.to(DEV), eps, out_dtype, **kw)
            assert (s.double().cpu() - new).abs().max() <= 1e-5 * new.abs().max()
            assert (got is None) == (out_dtype is None)
            if got is not None:
                assert got.dtype == out_dtype and (got.double().cpu() - new).abs().max() <= (1e-5 if out_dtype == torch.float32 else 1e-2) * new.abs().max()
        for taps in (1, 2, 4, 7):
            w = torch.randn(taps, H, generator=g)
            slots = torch.arange(T, dtype=torch.int32).flip(0).contiguous() + 1
            old = torch.randn(T + 2, max(4, (taps - 1) * H + 4), generator=g)
            state, s = old.clone().to(DEV), x.clone().to(DEV)
            got = ops.post_add(first.to(DEV), s, gain.to(DEV), eps, torch.float32, conv=(w.to(DEV), state, slots.to(DEV)), **kw)
            for t in range(T):
                past = old[slots[t], :(taps - 1) * H].double().view(taps - 1, H)
                rows = torch.cat((past, new[t:t + 1]))
                want = new[t] + (w.double() * rows).sum(0)
                assert (got[t].double().cpu() - want).abs().max() <= 2e-5 * want.abs().max()
                assert (state[slots[t], :(taps - 1) * H].double().cpu() - rows[1:].reshape(-1)).abs().max() <= 1e-5 * new.abs().max() if taps > 1 else True
            assert torch.equal(state[:, (taps - 1) * H:].cpu(), old[:, (taps - 1) * H:]) and torch.equal(state[0].cpu(), old[0])


@pytest.mark.parametrize("R,top,groups,keep", [(1, 1, 1, 1), (6, 2, 3, 2), (16, 4, 4, 3), (64, 8, 64, 8), (130, 5, 13, 2), (8, 8, 4, 4)])
def test_experts_from_the_best_groups_with_their_scores_as_weights(R, top, groups, keep):
    from ullm_amd.kernels import ops
    g = torch.Generator().manual_seed(R)
    T, H = 12, 40
    logits = torch.randn(T, R, generator=g) * 2
    logits[0] = 0.0                                      # a row of ties: the lower indices are taken
    s = torch.softmax(logits.double(), -1)
    order = torch.tensor([plain.choose_experts(r, top, groups, keep)[0] for r in s])
    ids, weights = ops.moe_route(logits.to(DEV), None, top, groups=groups, keep=keep, raw=True)
    assert torch.equal(ids.cpu().long(), order) and (weights.double().cpu() - torch.gather(s, 1, order)).abs().max() <= 1e-6
    ids, weights = ops.moe_route(logits.to(DEV), None, top, groups=groups, keep=keep, weight_scale=2.0)
    picked = torch.gather(s, 1, order)
    assert (weights.double().cpu() - 2 * picked / picked.sum(-1, keepdim=True)).abs().max() <= 1e-5
    # the product and the routing in one kernel, for few and for many rows
    w = torch.randn(R, H, generator=g) * 0.25
    for rows in (T, 600):
        x = torch.randn(rows, H, generator=g).to(torch.bfloat16)
        s = torch.softmax(x.double() @ w.double().T, -1)
        both = [plain.choose_experts(r, top, groups, keep) for r in s]
        clear, order = torch.tensor([m > 1e-4 for _, m in both]), torch.tensor([p for p, _ in both])
        assert clear.float().mean() > 0.8
        for dtype in (torch.float32, torch.bfloat16):
            ids, weights = ops.moe_router(x.to(DEV, dtype), w.to(DEV), None, top, groups=groups, keep=keep, raw=True)
            assert torch.equal(ids.cpu().long()[clear], order[clear])
            assert (weights.double().cpu() - torch.gather(s, 1, order))[clear].abs().max() <= 1e-4


@pytest.mark.parametrize("T", [1, 9, 200])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_gate_per_value_behind_the_product_per_head(T, dtype):
    from ullm_amd.kernels import ops
    g = torch.Generator().manual_seed(T)
    heads, K, N = 3, 24, 20
    x, w = torch.randn(T, heads, K + 8, generator=g).to(dtype), (torch.randn(heads, K, N, generator=g) * 0.2).to(dtype)
    wide = torch.randn(T, heads * N + 4, generator=g).to(dtype)
    out = torch.empty(T, heads, N, dtype=dtype, device=DEV)
    ops.head_linear(x.to(DEV)[:, :, :K], w.to(DEV), out=out, gate=wide.to(DEV)[:, 4:])
    want = torch.stack([x[:, h, :K].double() @ w[h].double() for h in range(heads)], 1) * torch.sigmoid(wide[:, 4:].double()).view(T, heads, N)
    assert (out.double().cpu() - want).abs().max() <= (1e-5 if dtype == torch.float32 else 1.5e-2) * want.abs().max()
