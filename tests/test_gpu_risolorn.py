"""Risolorn in the framework against the plain implementation (``plain_risolorn``, 64-bit): each mechanism's kernels alone
and as one-layer models; the stream after every layer; whole prompts; a prompt and then token by token, also from the
very first token; portions down to two tokens; unequal requests in one batch, in a pool and slots that are used again; long
decoding while chunks pass and pages return; scores scaled so that single keys just inside or outside a chunk, or the sink,
decide a row; memories that carry a token hundreds of steps; sizes that differ wherever they can, also values that make
things equal or one; many requests in one captured step; greedy generation through the entry point.
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

import plain_risolorn as plain
from gpu_util import DEV, paged_cache, table_tensor

pytestmark = pytest.mark.gpu

REL = {"float32": 3e-5, "bfloat16": 3e-2}
CLOSE_CALL = 0.02
# bfloat16 bounds (median, 85th of 100 rows, largest row ahead of the first close call)
BF16_BOUNDS = {"B": (4e-2, 1e-1, 0.5)}


def moe(experts, top, ff, groups=None):
    r = dict(experts=experts, top=top)
    if groups:
        r["groups"] = dict(count=groups[0], keep=groups[1])
    return dict(kind="moe", router=r, expert=dict(ff=ff))


def att(heads, kv, dim, vdim, scale, chunk, dims=0, base=1000.0, scaling=(4.0, 64, 8.0, 0.5), mlp=None):
    m = dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=scale)
    if chunk:
        m["mask"] = dict(size=chunk)
    if dims:
        m["rot"] = dict(base=base, dims=dims)
        if scaling:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return dict(type="attention", mixer=m, mlp=mlp)


def delta(heads, kv, dim, vdim, conv=3, mlp=None):
    return dict(type="delta", mixer=dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, conv=conv), mlp=mlp)


def mlstm(heads, dim, vdim, cap=8.0, mlp=None):
    return dict(type="mlstm", mixer=dict(heads=heads, dim=dim, vdim=vdim, gate_cap=cap), mlp=mlp)


def config(width, vocab, layers, eps=1e-5, scale=1.0, logit_scale=1.0):
    return dict(architecture="Risolorn", vocab=vocab, width=width, norm=dict(eps=eps), embedding=dict(scale=scale), logit_scale=logit_scale,
                layers=layers)


# A: every kind of layer twice, in another order each time, two chunk sizes, layers without a feed-forward
CFG_A = config(48, 131, [delta(6, 2, 16, 24, 4, moe(8, 3, 20, (4, 2))), att(6, 2, 16, 24, 0.4, 21, 8, mlp=moe(6, 2, 12, (2, 1))), mlstm(5, 12, 20, mlp=None),
                         mlstm(2, 24, 8, 15.0, moe(5, 3, 16)), delta(4, 4, 24, 8, 2, None), att(4, 4, 24, 8, 0.3, 33, 24, 50.0, None, moe(9, 2, 8, (3, 2)))],
               scale=0.7, logit_scale=0.6)
# B: values that make things equal or one, and sizes that no 16-byte access fits: one head, one channel, one expert, all
# experts, groups of one, one tap, five taps, a chunk of one, no chunk, no rotation
CFG_B = config(41, 97, [delta(3, 3, 6, 10, 1, moe(4, 4, 9, (1, 1))), att(1, 1, 6, 10, 0.5, 1, mlp=moe(1, 1, 14)), mlstm(1, 1, 7, 1.0, moe(6, 2, 7, (6, 2))),
                        delta(5, 1, 10, 1, 5, None), att(3, 3, 10, 6, 0.4, 0, 2, 30.0, (1.0, 10, 2.0, 2.0), moe(3, 1, 33)), mlstm(3, 13, 1, 3.0, None)])
# C: heads of 64 to 256 channels, more value than key channels and fewer, cached heads of 128 and 256 dims, a chunk shorter than a page
CFG_C = config(64, 211, [delta(4, 2, 128, 64, 4, moe(16, 4, 16, (4, 3))), att(4, 2, 128, 64, 0.09, 5, 64, mlp=moe(8, 2, 24)), mlstm(2, 64, 128, 15.0, None),
                         att(2, 1, 200, 40, 0.07, 48, 100, mlp=None), delta(2, 2, 200, 16, 3, None), mlstm(1, 160, 24, 10.0, moe(6, 2, 24, (3, 2)))], eps=1e-6, scale=0.5)
# W: scores of many units in chunks of 33: a row's weight lies on one or two keys or on the sink
CFG_W = config(32, 64, [att(2, 1, 16, 16, 1.5, 33, 4), att(4, 2, 16, 8, 1.2, 48, 16, 20.0, None)])
CFG_ATT = config(32, 64, [att(4, 2, 8, 8, 0.35, 12, 4)])
CFG_DELTA = config(32, 64, [delta(4, 2, 32, 8, 4)])
CFG_MLSTM = config(32, 64, [mlstm(2, 8, 8)])
CFG_MOE = config(32, 64, [att(1, 1, 8, 8, 0.3, 10, mlp=moe(12, 3, 8, (4, 2)))])
CFG_M = config(32, 50, [mlstm(2, 32, 64, 9.0, moe(8, 2, 16, (4, 2))), delta(8, 2, 32, 64, 4, None), att(4, 2, 32, 32, 0.2, 6, 8, mlp=None)])

MODELS = {"A": (CFG_A, 1), "B": (CFG_B, 2), "C": (CFG_C, 3), "W": (CFG_W, 4), "M": (CFG_M, 6), "att": (CFG_ATT, 7), "delta": (CFG_DELTA, 8),
          "mlstm": (CFG_MLSTM, 9), "moe": (CFG_MOE, 10)}


def made_weights(name):
    cfg, seed = MODELS[name]
    w = plain.random_weights(cfg, seed)
    if name == "W":
        for t in ("l0.mix.q", "l0.mix.k", "l1.mix.q", "l1.mix.k"):
            w[t] = (w[t].float() * 2).to(torch.bfloat16)
        for t in ("l0.mix.sink", "l1.mix.sink"):
            w[t] = (6 + 3 * w[t].float()).to(torch.bfloat16)
    if name in ("delta", "mlstm"):                        # slow memories: a token is still there hundreds of steps later
        if name == "delta":
            w["l0.mix.A_log"] -= 4
            w["l0.norm1.b"] += 1                          # and weak writes: later keys do not write over a first one
            w["l0.mix.b"] -= 0.15
        else:
            w["l0.mix.f.b"] += 3
    return w


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """{name: (folder, config, 64-bit weights)}; the folders hold bfloat16 tensors under the design's names."""
    out = {}
    for name, (cfg, _) in MODELS.items():
        d = tmp_path_factory.mktemp(f"risolorn{name}")
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
    if dtype == "float32" and rows is None and np.abs(got - want).max() > REL[dtype] * np.abs(want).max():
        # a row that is ill-conditioned in itself (one value over its own magnitude, next to zero): four times what the plain
        # implementation loses there in 32-bit
        _, cfg, w = models[name]
        narrow = plain.forward({k: v.float() for k, v in w.items()}, cfg, list(toks)).numpy()
        over = np.abs(got - want).max(-1) > np.maximum(REL[dtype] * np.abs(want).max(), 4 * np.abs(narrow - want).max(-1))
        assert not over.any(), np.nonzero(over)
        return
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
ALONE = [(n, d) for n in ("att", "delta", "mlstm", "moe") for d in ("float32", "bfloat16")]


@pytest.mark.parametrize("name,dtype", BIG + ALONE)
def test_whole_prompts(replayers, models, name, dtype):
    rep = replayers(name, dtype)
    for i, n in enumerate((1, 2, 15, 16, 17, 90)):
        toks = tokens(models[name][1]["vocab"], n, 10 + i)
        agree(models, name, toks, run(rep, "r", toks, [n]), dtype)


@pytest.mark.parametrize("name,dtype", [("delta", "float32"), ("mlstm", "float32"), ("mlstm", "bfloat16"), ("A", "float32"), ("C", "float32")])
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
    """Layer by layer in 32-bit: the stream once what the layer left pending is added."""
    from ullm_amd.engine.loading import load_model
    from ullm_amd.engine.runner import ModelRunner, StepEntry
    from ullm_amd.kernels import ops
    d, cfg, w = models[name]
    toks = tokens(cfg["vocab"], 50, 3)
    want = []
    plain.forward(w, cfg, toks, want)
    _, model, env = load_model(d, "float32", DEV, context_len=64)
    runner = ModelRunner(model, env, page_size=16, num_pages=4, max_requests=1, use_graphs=False)
    rc = runner.cache.admit("r")
    assert runner.cache.reserve(rc, len(toks))
    ctx, _ = runner.build_context([StepEntry(rc, toks, [])])
    stream = ops.embedding(ctx.token_ids, model.embedding, scale=model.plan.embedding_scale)
    pending = None
    for i, (block, cache_id) in enumerate(model.run_order):
        stream, pending = model.blocks[block].forward(stream, pending, ctx, runner.caches.get(cache_id))
        after = (stream.double() + pending.mult * pending.joined().double()).cpu()
        assert pending.post is None and (after - want[i]).abs().max() <= 3e-5 * want[i].abs().max(), i


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
    """140 requests a step, one token each, nine steps (chunks pass): captured steps that are replayed against the same steps
    run eagerly and against the plain implementation."""
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
def test_long_decoding_while_chunks_pass_and_pages_return(replayers, models, dtype):
    """190 tokens one by one through captured steps: chunk after chunk is over and its pages go back to the pool, memories
    carry on; a second request then takes the pages and the slot again."""
    rep = replayers("A", dtype, max_tokens=192)
    toks = tokens(models["A"][1]["vocab"], 190, 40)
    agree(models, "A", toks, run(rep, "r", toks, [3]), dtype)
    other = tokens(models["A"][1]["vocab"], 100, 41)
    agree(models, "A", other, run(rep, "s", other, [60]), dtype)


def test_a_chunk_s_pages_are_free_for_others_while_its_request_goes_on(replayers, models):
    rep = replayers("att", "float32", max_tokens=192)
    cache = rep.runner.cache
    toks = tokens(64, 150, 45)
    for i, t in enumerate(toks):
        rep.step({"step": i, "entries": [{"id": "r", "tokens": [t], "want": []}], "end": []})
        # chunks of 12 positions in pages of 16: never more than two pages behind a committed step
        assert cache.allocators[0].num_pages - cache.num_free_pages(0) <= 2
    rep.step({"step": 999, "entries": [], "end": ["r"]})


EDGE_CUTS = [(200,), (120,), (17, 64, 2, 31, 2, 30), (33, 33, 1, 1, 47, 47, 2, 16), (32, 1, 1, 1, 66, 34), (98, 2, 2, 2)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cuts", EDGE_CUTS)
def test_single_keys_and_the_sink_decide(replayers, models, dtype, cuts):
    """Scores of many units: a row's weight lies on one or two keys or on the sink, in portions and for single tokens: a chunk
    one position off, a key lost at a page's border or a sink left out moves the row."""
    toks = tokens(models["W"][1]["vocab"], 200, 42)
    want, _ = oracle_and_gaps(models, "W", toks)
    got = run(replayers("W", dtype), "r", toks, cuts)
    if dtype == "float32":
        close(got, want, dtype)
    else:
        err = np.abs(got - want).max(-1) / np.abs(want).max()
        assert np.median(err) < 4e-2 and err.max() < 0.35, (np.median(err), err.max())


def test_edges_and_sinks_decide_rows_in_the_peaked_model(models):
    """The plain implementation itself: with a chunk one position longer or shorter, chunks counted from another position, or
    without sinks, several rows move by far more than the bounds above."""
    toks = tokens(64, 200, 42)
    _, cfg, w = models["W"]
    base = plain.forward(w, cfg, toks)

    def moved(change=None, weights=w, seen=None):
        c, keep = copy.deepcopy(cfg), plain.same_chunk
        if change:
            change(c["layers"])
        if seen:
            plain.same_chunk = seen
        try:
            m = (plain.forward(weights, c, toks) - base).abs().max(-1).values / base.abs().max()
        finally:
            plain.same_chunk = keep
        return int((m > 0.03).sum())
    for layer, size in ((0, 32), (0, 34), (1, 47), (1, 49)):
        assert moved(lambda L: L[layer]["mixer"]["mask"].update(size=size)) >= 3, (layer, size)
    keep = plain.same_chunk

    def late(T, size):                                   # chunks that begin a position late
        m = torch.zeros(T, T, dtype=torch.bool)
        m[1:, 1:] = keep(T - 1, size)
        m[0, 0] = True
        return m
    assert moved(seen=late) >= 3
    for layer in (0, 1):
        assert moved(weights={**w, f"l{layer}.mix.sink": w[f"l{layer}.mix.sink"] - 100}) >= 20, layer


@pytest.mark.parametrize("name", ["delta", "mlstm"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cuts", [(300,), (1, 150, 2, 100), (290,)])
def test_a_token_hundreds_of_steps_back_is_still_there(replayers, models, name, dtype, cuts):
    """Slow memories still hold the first token after 300 steps: the last logits move when the first token is another one (in
    the plain implementation), and the framework follows."""
    _, cfg, _ = models[name]
    toks = tokens(cfg["vocab"], 300, 44)
    other = [(toks[0] + 1) % cfg["vocab"]] + toks[1:]
    base, changed = oracle_and_gaps(models, name, toks)[0], oracle_and_gaps(models, name, other)[0]
    assert np.abs(base[-1] - changed[-1]).max() > 2e-4 * np.abs(base).max()
    got = run(replayers(name, dtype), "r", toks, cuts)
    agree(models, name, toks, got, dtype)
    if dtype == "float32":
        got_other = run(replayers(name, dtype), "r", other, cuts)
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
    config, _ = parse_random_weights("risolorn-2048")
    cfg, model = build_model(config)
    assert cfg.hidden_size == 2048 and len(model.blocks) == 8 and {L.type for L in cfg.layers} == {"delta", "mlstm", "attention"}


# ------------------------------------------------------------------------------------------- kernels alone

def step_context(lens, starts=None, slots=None):
    """What the kernels read of a step with entries of these lengths (slots in another order than the entries)."""
    from ullm_amd.parts.base import StepShape
    from ullm_amd.parts.memory import plan_memory_chunks
    q = np.concatenate(([0], np.cumsum(lens))).astype(np.int32)
    starts = starts or [0] * len(lens)
    to = lambda a: torch.from_numpy(np.ascontiguousarray(np.asarray(a, dtype=np.int32))).to(DEV)      # noqa: E731
    chunks = plan_memory_chunks(StepShape(tuple(lens), tuple(starts)))
    chunks.arrays = {k: to(v) for k, v in chunks.arrays.items()}
    return SimpleNamespace(chunks=chunks, q_start=to(q), token_entry=to(np.repeat(np.arange(len(lens)), lens)), num_entries=len(lens),
                           entry_slot=to(slots if slots is not None else np.arange(len(lens))[::-1] + 1),
                           positions=to(np.concatenate([s + np.arange(n) for s, n in zip(starts, lens)])),
                           decode_only=all(n == 1 for n in lens), max_q_len=max(lens))


STEPS = ([37, 1, 70], [2, 18, 1], [1, 1, 1], [16, 2, 1], [1, 1, 1])
LONG_STEPS = ([301, 2, 1], [1, 1500, 270], [5, 1, 1])


def over_steps(seqs, steps, call):
    """Three requests' rows through the steps: ``call(ctx, the step's rows of every tensor of seqs)`` -> tensors of rows; returns
    each of them per request."""
    at, got = [0, 0, 0], [[], [], []]
    for lens in steps:
        ctx = step_context(lens)
        rows = [torch.cat([s[k][a:a + n] for s, a, n in zip(seqs, at, lens)]).to(DEV) for k in range(len(seqs[0]))]
        outs = [o.double().cpu() for o in call(ctx, *rows)]
        row = 0
        for i, n in enumerate(lens):
            got[i].append([o[row:row + n] for o in outs])
            row += n
            at[i] += n
    return [[torch.cat([s[k] for s in g]) for k in range(len(g[0]))] for g in got]


def untouched(state, off, n):
    """Values around the three requests' rows 1 .. 3 of a state that was filled with 3 ahead of and behind its part."""
    s = state.cpu()
    return bool((s[:, :off] == 3.0).all() and (s[:, off + n:] == 3.0).all() and (s[0, off:off + n] == 0).all() and (s[4, off:off + n] == 0).all())


@pytest.mark.parametrize("heads,kv,N,P", [(1, 1, 1, 1), (4, 2, 8, 12), (3, 3, 13, 7), (6, 2, 32, 40), (2, 2, 40, 64), (4, 1, 64, 16), (2, 1, 128, 128), (2, 2, 130, 20),
                                          (1, 1, 256, 33), (2, 1, 300, 8), (1, 1, 512, 5)])
@pytest.mark.parametrize("rule", ["delta", "sum"])
def test_the_matrix_memory_alone(heads, kv, N, P, rule):
    """Three requests in five steps of portions and single tokens, q and k columns of wider rows, the memories between other values."""
    from ullm_amd.kernels import ops
    g = torch.Generator().manual_seed(heads * 1000 + N + P)
    seqs = []
    for i in range(3):
        n = sum(s[i] for s in STEPS)
        k = torch.nn.functional.normalize(torch.randn(n, kv, N, generator=g), dim=-1).reshape(n, kv * N)
        seqs.append((torch.randn(n, kv * N, generator=g), k, torch.randn(n, heads * P, generator=g), 0.5 + 0.5 * torch.rand(n, heads, generator=g),
                     torch.rand(n, heads, generator=g)))
    off, size = 4, heads * N * P + (heads * N if rule == "sum" else 0)
    state = torch.full((5, off + size + 3), 3.0, device=DEV)
    state[:, off:off + size] = 0.0

    def call(ctx, q, k, v, keep, take):
        wide = torch.cat((v, q, k), dim=1)
        gates = torch.stack((keep, take), dim=1)
        o, n = ops.matrix_memory(wide[:, v.shape[1]:v.shape[1] + kv * N], wide[:, v.shape[1] + kv * N:], wide[:, :v.shape[1]], gates[:, 0], gates[:, 1],
                                 ops.MEMORY_DELTA if rule == "delta" else ops.MEMORY_SUM, state, off, ctx, heads, kv, N, P, ctx.chunks, q_scale=0.7,
                                 norm_off=off + heads * N * P)
        return (o,) if n is None else (o, n)
    got = over_steps(seqs, STEPS, call)
    for (q, k, v, keep, take), out in zip(seqs, got):
        T = q.shape[0]
        q, k, v = q.double().view(T, kv, N) * 0.7, k.double().view(T, kv, N), v.double().view(T, heads, P)
        want, norm = torch.zeros(T, heads, P, dtype=torch.float64), torch.zeros(T, heads, dtype=torch.float64)
        for h in range(heads):
            qh, kh = q[:, h // (heads // kv)], k[:, h // (heads // kv)]
            if rule == "delta":
                want[:, h] = plain.delta_rule(qh, kh, v[:, h], keep[:, h].double(), take[:, h].double())
            else:
                S, n = torch.zeros(N, P, dtype=torch.float64), torch.zeros(N, dtype=torch.float64)
                for t in range(T):
                    S = keep[t, h].double() * S + take[t, h].double() * torch.outer(kh[t], v[t, h])
                    n = keep[t, h].double() * n + take[t, h].double() * kh[t]
                    want[t, h], norm[t, h] = qh[t] @ S, n @ qh[t]
        assert (out[0].view(T, heads, P) - want).abs().max() <= 5e-6 * want.abs().max()
        if rule == "sum":
            assert (out[1] - norm).abs().max() <= 5e-6 * norm.abs().max()
    assert untouched(state, off, size)


def test_the_matrix_memory_of_many_entries(heads=8, N=40, P=128):
    """Steps with entries enough that single tokens take slices of 64 value channels."""
    from ullm_amd.kernels import ops
    g = torch.Generator().manual_seed(3)
    B = 140
    for rule in (ops.MEMORY_DELTA, ops.MEMORY_SUM):
        state = torch.zeros(B, heads * N * (P + 1), device=DEV)
        S, n = torch.zeros(B, heads, N, P).double(), torch.zeros(B, heads, N).double()
        for lens in ([1] * B, [1] * B, [3] + [1] * (B - 1), [1] * B):
            ctx = step_context(lens, slots=list(range(B)))
            T = sum(lens)
            q, k, v = torch.randn(T, heads * N, generator=g), torch.nn.functional.normalize(torch.randn(T, heads, N, generator=g), dim=-1).view(T, -1), torch.randn(T, heads * P, generator=g)
            keep, take = torch.rand(T, heads, generator=g), torch.rand(T, heads, generator=g)
            o, norm = ops.matrix_memory(q.to(DEV), k.to(DEV), v.to(DEV), keep.to(DEV), take.to(DEV), rule, state, 0, ctx, heads, heads, N, P, ctx.chunks, norm_off=heads * N * P)
            want, want_n = torch.zeros(T, heads, P).double(), torch.zeros(T, heads).double()
            t = 0
            for b, L in enumerate(lens):
                for _ in range(L):
                    qq, kk, vv, g1, b1 = q[t].double().view(heads, N), k[t].double().view(heads, N), v[t].double().view(heads, P), keep[t].double(), take[t].double()
                    S[b] *= g1[:, None, None]
                    u = b1[:, None] * (vv - (S[b] * kk[:, :, None]).sum(1) if rule == ops.MEMORY_DELTA else vv)
                    S[b] += kk[:, :, None] * u[:, None, :]
                    n[b] = g1[:, None] * n[b] + b1[:, None] * kk
                    want[t], want_n[t] = (S[b] * qq[:, :, None]).sum(1), (n[b] * qq).sum(1)
                    t += 1
            assert (o.double().cpu().view(T, heads, P) - want).abs().max() <= 5e-6 * want.abs().max()
            if rule == ops.MEMORY_SUM:
                assert (norm.double().cpu() - want_n).abs().max() <= 5e-6 * want_n.abs().max()
        assert (state[:, :heads * N * P].double().cpu().view(B, heads, N, P) - S).abs().max() <= 5e-6 * S.abs().max()


@pytest.mark.parametrize("heads,kv,N,P,taps", [(1, 1, 1, 1, 1), (4, 2, 8, 12, 4), (3, 3, 13, 70, 3), (6, 2, 32, 40, 2), (2, 1, 128, 64, 4), (2, 2, 200, 16, 4), (1, 1, 20, 300, 9)])
@pytest.mark.parametrize("steps", [STEPS, LONG_STEPS], ids=["short", "long"])
def test_what_stands_ahead_of_the_delta_rule(heads, kv, N, P, taps, steps):
    """Convolution, silu, unit queries and keys, decays and write strengths, the carried inputs between other values."""
    from ullm_amd.kernels import ops
    g = torch.Generator().manual_seed(heads + N + P + taps)
    channels = 2 * kv * N + heads * P
    w = torch.randn(channels, taps, generator=g) / math.sqrt(taps)
    a_log, dt_bias = torch.log(torch.rand(heads, generator=g) * 3 + 0.01), torch.randn(heads, generator=g)
    seqs = [(torch.randn(sum(s[i] for s in steps), channels, generator=g), 4 * torch.randn(sum(s[i] for s in steps), 2 * heads, generator=g)) for i in range(3)]
    off, size = 4, (taps - 1) * channels
    state = torch.full((5, off + size + 3), 3.0, device=DEV)
    state[:, off:off + size] = 0.0
    a_rate = torch.exp(a_log.double()).float().to(DEV)

    def call(ctx, x, raw):
        wide = torch.cat((raw[:, :heads], x, raw[:, heads:]), dim=1)
        out, gates = ops.delta_prepare(wide[:, heads:heads + channels], w.t().contiguous().to(DEV), wide[:, :heads], wide[:, heads + channels:], a_rate,
                                       dt_bias.to(DEV), state, off, ctx, heads, kv, N, P, 0.3)
        return out, gates[:, 0], gates[:, 1]
    for (x, raw), (rows, keep, take) in zip(seqs, over_steps(seqs, steps, call)):
        T = x.shape[0]
        y = plain.silu(plain.causal_conv(x.double(), w.double()))
        q, k, v = y[:, :kv * N].view(T, kv, N), y[:, kv * N:2 * kv * N].view(T, kv, N), y[:, 2 * kv * N:]
        want = torch.cat((plain.unit(q).reshape(T, -1) * 0.3, plain.unit(k).reshape(T, -1), v), dim=1)
        assert (rows - want).abs().max() <= 5e-6 * want.abs().max()
        assert (take - torch.sigmoid(raw[:, :heads].double())).abs().max() <= 2e-6
        z = raw[:, heads:].double() + dt_bias.double()
        assert (keep - torch.exp(-torch.exp(a_log.double()) * plain.softplus(z))).abs().max() <= 3e-6
    assert untouched(state, off, size)
    if taps > 1:
        last = torch.cat((torch.zeros(taps - 1, channels), seqs[0][0]))[-(taps - 1):]
        assert torch.equal(state[3, off:off + size].view(taps - 1, channels).cpu(), last)


@pytest.mark.parametrize("heads,cap", [(1, 15.0), (5, 2.0), (70, 30.0)])
@pytest.mark.parametrize("steps", [STEPS, LONG_STEPS], ids=["short", "long"])
def test_exponential_gates_alone(heads, cap, steps):
    """Portions of one to 1500 tokens: the running maximum across lanes, waves and rounds of a block, and from step to step."""
    from ullm_amd.kernels import ops
    g = torch.Generator().manual_seed(heads)
    b_i, b_f = torch.randn(heads, generator=g), 3 + torch.randn(heads, generator=g)
    seqs = []
    for i in range(3):
        n = sum(s[i] for s in steps)
        raw = 6 * torch.randn(n, 2 * heads, generator=g)
        raw[::50] += 10                                   # now and then a token that overrides what came before
        seqs.append((raw,))
    off = 2
    state = torch.full((5, off + heads + 3), 3.0, device=DEV)
    state[:, off:off + heads] = 0.0

    def call(ctx, raw):
        gates = ops.exp_gates(raw[:, :heads], raw[:, heads:], b_i.to(DEV), b_f.to(DEV), cap, state, off, ctx)
        return gates[:, 0], gates[:, 1], gates[:, 2]
    for (raw,), (keep, take, floor) in zip(seqs, over_steps(seqs, steps, call)):
        i = cap * torch.tanh((raw[:, :heads].double() + b_i.double()) / cap)
        f = plain.logsigmoid(cap * torch.tanh((raw[:, heads:].double() + b_f.double()) / cap))
        m = torch.zeros(heads, dtype=torch.float64)
        for t in range(raw.shape[0]):
            top = torch.maximum(f[t] + m, i[t])
            for got, want in ((keep[t], torch.exp(f[t] + m - top)), (take[t], torch.exp(i[t] - top)), (floor[t], torch.exp(-top))):
                assert (got - want).abs().max() <= 2e-5 * want.abs().max() + 1e-12, t
            m = top
    assert untouched(state, off, heads)


@pytest.mark.parametrize("parts,size", [(1, 1), (3, 20), (4, 64), (2, 1030)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_outputs_over_their_normaliser(parts, size, dtype):
    from ullm_amd.kernels import ops
    g = torch.Generator().manual_seed(size)
    T, eps = 9, 1e-5
    o, gate, gain = torch.randn(T, parts * size, generator=g), torch.randn(T, parts * size, generator=g), 1 + 0.2 * torch.randn(parts * size, generator=g)
    den, gates = torch.randn(T, parts, generator=g), torch.rand(T, 3, parts, generator=g)
    den[0], gates[0, 2] = 0.0, 0.0                        # nothing but the constant divides
    got = ops.gated_unit_norm(o.to(DEV), gate.to(DEV), gain.to(DEV), eps, parts, ops.GATE_SIGMOID, dtype, den=den.to(DEV), least=gates.to(DEV)[:, 2])
    y = o.double().view(T, parts, size) / (torch.maximum(den.double().abs(), gates[:, 2].double()) + 1e-6)[..., None]
    want = plain.over_rms(y, eps).view(T, -1) * gain.double() * torch.sigmoid(gate.double())
    assert (got.double().cpu() - want).abs().max() <= (1e-5 if dtype == torch.float32 else 1e-2) * want.abs().max()


@pytest.mark.parametrize("H", [1, 8, 41, 300, 2048])
def test_the_stream_squashed(H):
    """A branch, a stack of partial sums or nothing joins the stream; chosen rows only; both dtypes on either side."""
    from ullm_amd.kernels import ops
    g = torch.Generator().manual_seed(H)
    T = 9
    x, alpha, gain, shift = torch.randn(T, H, generator=g), torch.tensor(0.6), torch.randn(H, generator=g), torch.randn(H, generator=g)
    stack = torch.randn(3, T, H, generator=g)
    rows = torch.tensor([7, 0, 7, 3], dtype=torch.int32)
    for dtype in (torch.float32, torch.bfloat16):
        for branch in (None, stack[0].to(dtype), stack.to(dtype)):
            y = 0 if branch is None else 0.5 * (branch.double() if branch.dim() == 2 else branch.double().sum(0))
            new = x.double() + y
            want = torch.tanh(0.6 * new) * gain.double() + shift.double()
            for out_dtype in (torch.float32, torch.bfloat16):
                tol = (2e-6 if out_dtype == torch.float32 else 1e-2) * want.abs().max()
                s = x.clone().to(DEV)
                args = [None if branch is None else branch.to(DEV), s, alpha.to(DEV), gain.to(DEV), shift.to(DEV), out_dtype]
                got = ops.add_tanh(*args, rows=rows.to(DEV), mult=0.5)
                assert torch.equal(s.cpu(), x) and (got.double().cpu() - want[rows.long()]).abs().max() <= tol
                got = ops.add_tanh(*args, mult=0.5)
                assert got.dtype == out_dtype and (got.double().cpu() - want).abs().max() <= tol
                assert (s.double().cpu() - new).abs().max() <= 1e-6 * new.abs().max()


@pytest.mark.parametrize("nq,nkv,hd", [(3, 3, 32), (8, 2, 64), (6, 1, 96), (4, 2, 128), (2, 2, 256), (40, 2, 32), (4, 2, 48), (5, 5, 10)])
@pytest.mark.parametrize("chunk", [1, 5, 16, 32, 37, 64, 100, 1000])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_attention_in_chunks_alone(nq, nkv, hd, chunk, dtype):
    """Decoded tokens beside portions, at positions around the chunks' edges; pages wholly before a chunk are not held and
    unused rows of the pools hold NaN; with and without a sink."""
    from ullm_amd.kernels import ops
    from ullm_amd.parts.attention import plan_attention_step
    from ullm_amd.parts.base import StepShape
    g = torch.Generator().manual_seed(nq * 1000 + hd + chunk)
    totals, lens = [150, 38, 97, 1, 70, 128, 201], [1, 1, 60, 1, 35, 128, 1]
    starts = [t - n for t, n in zip(totals, lens)]
    P = 16
    ks = [torch.randn(t, nkv, hd, generator=g).to(dtype) for t in totals]
    vs = [torch.randn(t, nkv, hd, generator=g).to(dtype) for t in totals]
    k_pool, v_pool, tables = paged_cache(ks, vs, P, dtype, DEV, seed=1)
    for table, s in zip(tables, starts):
        for i in range(s // chunk * chunk // P):          # given back when the chunk was over
            k_pool[table[i]], v_pool[table[i]] = float("nan"), float("nan")
            table[i] = -1
    ctx = step_context(lens, starts)
    group = SimpleNamespace(block_table=table_tensor(tables, DEV), page_size=P)
    q = (2 * torch.randn(sum(lens), nq, hd, generator=g)).to(dtype)
    sink = 2 * torch.randn(nq, generator=g)
    plan = plan_attention_step(StepShape(tuple(lens), tuple(starts)))
    plan.arrays = {k: torch.from_numpy(v).to(DEV) for k, v in plan.arrays.items()}
    for sinks in (None, sink):
        want, row = [], 0
        for i, n in enumerate(lens):
            seen = plain.same_chunk(totals[i], chunk)[starts[i]:]
            o = torch.zeros(n, nq, hd, dtype=torch.float64)
            for h in range(nq):
                kvh = h // (nq // nkv)
                s = ((q[row:row + n, h].double() @ ks[i][:, kvh].double().T) * hd ** -0.5).masked_fill(~seen, -math.inf)
                e = torch.exp(s)
                o[:, h] = e @ vs[i][:, kvh].double() / (e.sum(-1, keepdim=True) + (0 if sinks is None else math.exp(sinks[h].item())))
            want.append(o)
            row += n
        want = torch.cat(want).reshape(sum(lens), nq * hd)
        extra = {} if sinks is None else dict(sink=sinks.to(DEV), sink_log2=(sinks * math.log2(math.e)).to(DEV))
        got = ops.paged_attention(q.reshape(sum(lens), nq * hd).to(DEV), k_pool, v_pool, ctx, group, nq, nkv, hd, hd ** -0.5, -chunk, plan, **extra).double().cpu()
        assert torch.isfinite(got).all()
        err = (got - want).abs().max() / want.abs().max()
        assert err <= (2e-5 if dtype == torch.float32 else 1.5e-2), (sinks is None, float(err))


@pytest.mark.parametrize("hd", [32, 128])
@pytest.mark.parametrize("n", [1, 7, 40])
@pytest.mark.parametrize("chunk", [30, 64, 77])
def test_one_key_stands_out_at_a_chunk_s_edge(hd, n, chunk):
    """The last query's own chunk begins at `lo`; one key's score stands out by hundreds: seen at lo, lo + 1 and at a page's
    border, not seen at lo - 1."""
    from ullm_amd.kernels import ops
    from ullm_amd.parts.attention import plan_attention_step
    from ullm_amd.parts.base import StepShape
    g = torch.Generator().manual_seed(hd + n + chunk)
    S, P, nq, nkv = 3 * chunk - 5, 16, 4, 2
    lo = 2 * chunk
    direction = torch.nn.functional.normalize(torch.randn(hd, generator=g), dim=0)
    for target in (lo - 1, lo, lo + 1, (lo // P + 1) * P - 1, (lo // P + 1) * P, S - 1):
        k = torch.randn(S, nkv, hd, generator=g) * 0.1
        v = torch.randn(S, nkv, hd, generator=g)
        q = torch.randn(n, nq, hd, generator=g) * 0.1
        k[target], q[-1] = 30.0 * direction, 30.0 * direction
        for dtype in (torch.float32, torch.bfloat16):
            k_pool, v_pool, tables = paged_cache([k], [v], P, dtype, DEV, seed=target)
            ctx = step_context([n], [S - n])
            plan = plan_attention_step(StepShape((n,), (S - n,)))
            plan.arrays = {a: torch.from_numpy(b).to(DEV) for a, b in plan.arrays.items()}
            got = ops.paged_attention(q.reshape(n, -1).to(DEV, dtype), k_pool, v_pool, ctx, SimpleNamespace(block_table=table_tensor(tables, DEV), page_size=P),
                                      nq, nkv, hd, 1.0, -chunk, plan).float().cpu().view(n, nq, hd)[-1]
            away = max(float((got[h] - v[target, h // 2]).abs().max()) for h in range(nq))
            assert (away < 3e-2) == (target >= lo), (target, lo, dtype, away)


@pytest.mark.parametrize("R,top,groups,keep", [(1, 1, 1, 1), (6, 2, 3, 2), (16, 4, 4, 3), (64, 8, 64, 8), (130, 5, 13, 2), (8, 8, 4, 4), (12, 3, 2, 1)])
def test_experts_from_the_groups_with_the_best_two_scores(R, top, groups, keep):
    from ullm_amd.kernels import ops
    g = torch.Generator().manual_seed(R)
    T, H = 40, 40
    kw = dict(groups=groups, keep=keep, raw=True, group_top=2)
    for shift in (0.0, -1.5):                             # also where every choice score is negative
        logits, corr = torch.randn(T, R, generator=g) * 2, torch.randn(R, generator=g) * 0.4 + shift
        logits[0] = 0.0
        s = torch.sigmoid(logits.double())
        both = [plain.choose_experts(r, top, groups, keep) for r in s + corr.double()]
        clear, order = torch.tensor([m > 1e-5 for _, m in both]), torch.tensor([p for p, _ in both])
        ids, weights = ops.moe_route(logits.to(DEV), corr.to(DEV), top, ops.ROUTE_SIGMOID, **kw)
        assert clear.float().mean() > 0.8 and torch.equal(ids.cpu().long()[clear], order[clear])
        assert (weights.double().cpu() - torch.gather(s, 1, order))[clear].abs().max() <= 1e-6
        w = torch.randn(R, H, generator=g) * 0.25          # the product and the routing in one kernel, for few and for many rows
        for rows in (T, 600):
            x = torch.randn(rows, H, generator=g).to(torch.bfloat16)
            s = torch.sigmoid(x.double() @ w.double().T)
            both = [plain.choose_experts(r, top, groups, keep) for r in s + corr.double()]
            clear, order = torch.tensor([m > 1e-4 for _, m in both]), torch.tensor([p for p, _ in both])
            assert clear.float().mean() > 0.8
            ids, weights = ops.moe_router(x.to(DEV), w.to(DEV), corr.to(DEV), top, ops.ROUTE_SIGMOID, **kw)
            assert torch.equal(ids.cpu().long()[clear], order[clear])
            assert (weights.double().cpu() - torch.gather(s, 1, order))[clear].abs().max() <= 1e-4


def test_group_sums_and_group_maxima_choose_differently():
    from ullm_amd.kernels import ops
    z = torch.tensor([[3.0, -3.0, 1.0, 1.0]])             # the largest score's group has the smaller sum
    for group_top, want in ((1, 0), (2, 2)):
        ids, _ = ops.moe_route(z.to(DEV), None, 1, ops.ROUTE_SIGMOID, groups=2, keep=1, raw=True, group_top=group_top)
        assert ids.item() == want
