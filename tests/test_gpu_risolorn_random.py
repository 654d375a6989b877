"""Risolorn configurations drawn at random (width, order of layers, heads, key and value sizes, chunks, taps, gate caps,
rotations and their stretch, experts and groups, layers without a feed-forward) through the replayer: in 32-bit against the
plain 64-bit implementation, whole prompts, portions of drawn sizes followed by single tokens, and a schedule of up to four
live requests in a pool and slots that are used again; in bfloat16 the same schedules against the same logits, most rows to
rounding."""
import json
import os
import random

import numpy as np
import pytest
import torch
from safetensors.torch import save_file

import plain_risolorn as plain
from gpu_util import DEV
from test_gpu_kumudra_random import schedules, worst_error

pytestmark = pytest.mark.gpu


def drawn_mlp(rng):
    if rng.random() < 0.2:
        return None
    count = rng.choice([1, 1, 2, 3, 4, 8])
    experts = count * rng.choice([1, 2, 3, 4, 5])
    keep = rng.randint(1, count)
    return dict(kind="moe", router=dict(experts=experts, top=rng.randint(1, min(6, experts // count * keep)), groups=dict(count=count, keep=keep)),
                expert=dict(ff=rng.choice([4, 6, 8, 12, 16, 24, 40, 64, 100, 130])))


def drawn_layer(rng):
    kind = rng.choice(["delta", "mlstm", "attention"])
    kv = rng.choice([1, 1, 2, 3, 4])
    heads = kv * rng.choice([1, 2, 3, 4])
    dim = rng.choice([4, 8, 12, 16, 24, 32, 40, 64, 72, 96, 128, 160, 256])
    vdim = rng.choice([dim, dim, 4, 5, 8, 20, 64, 128])
    if kind == "delta":
        m = dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, conv=rng.choice([1, 2, 3, 4, 4, 5, 7]))
    elif kind == "mlstm":
        m = dict(heads=rng.choice([1, 2, 3, 5, 8]), dim=dim, vdim=vdim, gate_cap=rng.choice([1.0, 5.0, 15.0, 30.0]))
    else:
        dims = rng.choice([2, dim // 4 * 2, dim // 2 * 2])
        rot = dict(base=rng.choice([20.0, 1e4, 5e5]), dims=dims,
                   scaling=dict(factor=rng.choice([1.0, 2.0, 8.0, 40.0]), original=rng.choice([16, 64, 2048]), fast=rng.choice([4.0, 32.0]), slow=rng.choice([0.3, 1.0, 2.0])))
        m = dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=rng.choice([0.5, 1.0, 2.0]) * dim ** -0.5, mask=dict(size=rng.choice([1, 2, 5, 16, 17, 33, 48, 64, 150])), rot=rot)
    return dict(type=kind, mixer=m, mlp=drawn_mlp(rng))


def drawn_config(rng):
    return dict(architecture="Risolorn", vocab=rng.randint(40, 700), layers=[drawn_layer(rng) for _ in range(rng.randint(1, 6))], norm=dict(eps=rng.choice([1e-5, 1e-6, 1e-3])),
                width=rng.choice([20, 24, 32, 36, 40, 48, 50, 64, 72, 96, 100, 128, 160, 256]), embedding=dict(scale=rng.choice([0.3, 1.0, 2.0])),
                logit_scale=rng.choice([0.25, 1.0, 3.0]))


@pytest.mark.parametrize("seed", range(24))
def test_drawn_configurations(seed, tmp_path):
    from ullm_amd.replay import Replayer
    rng = random.Random(7300 + seed)
    cfg = drawn_config(rng)
    w = plain.random_weights(cfg, seed)
    with open(os.path.join(tmp_path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in w.items()}, os.path.join(tmp_path, "model.safetensors"))
    wide = {k: v.double() for k, v in w.items()}
    reqs = {f"r{i}": [rng.randrange(cfg["vocab"]) for _ in range(rng.randint(20, 110))] for i in range(6)}
    want, sharp, clear = {}, {}, {}
    for k, t in reqs.items():
        plain.MARGINS = []
        want[k] = plain.forward(wide, cfg, t).float().numpy()
        # rows before the first token whose choice nearly ties (32-bit sums may settle it otherwise, and every later row
        # sees that token through the states): only these are held to the 32-bit bound
        gaps = np.min([m.numpy() for m in plain.MARGINS], axis=0) if plain.MARGINS else np.full(len(t), np.inf)
        plain.MARGINS = None
        close_calls = np.nonzero(gaps < 1e-5)[0]
        sharp[k] = int(close_calls[0]) if len(close_calls) else len(t)
        calls = np.nonzero(gaps < 0.02)[0]
        clear[k] = int(calls[0]) if len(calls) else len(t)          # ahead of the first choice that rounding may move
    assert sum(sharp.values()) >= 0.4 * sum(len(t) for t in reqs.values()), ("near-ties leave too few rows to compare", sharp)
    narrow = {k: v.float() for k, v in w.items()}
    # what 32-bit sums alone do to this model (six times that, as the engine sums in another order), at least 5e-5
    bound = {k: max(5e-5, 6 * worst_error(plain.forward(narrow, cfg, t).numpy()[:sharp[k]], want[k][:sharp[k]])) if sharp[k] else 1.0
             for k, t in reqs.items()}
    state = rng.getstate()
    whole, cut, mixed = schedules(Replayer(str(tmp_path), "float32", 512, 16, DEV, max_requests=4), rng, reqs)
    n0 = sharp["r0"]
    for what, got in (("whole", whole), ("cut", cut)):
        assert worst_error(got[:n0], want["r0"][:n0]) <= bound["r0"], (what, worst_error(got[:n0], want["r0"][:n0]), bound["r0"])
    for k in reqs:
        assert worst_error(mixed[k][:sharp[k]], want[k][:sharp[k]]) <= bound[k], (k, worst_error(mixed[k][:sharp[k]], want[k][:sharp[k]]), bound[k])
    # bfloat16: the same schedules.  The bounds for the rows ahead of the first close call are multiples of what the plain
    # implementation loses when nothing but its sublayers' inputs are rounded to bfloat16, for the middle row and for 85 of
    # 100; behind it a row whose router picks another expert moves as a whole, and the rows behind it with it.
    rng.setstate(state)
    whole, cut, mixed = schedules(Replayer(str(tmp_path), "bfloat16", 512, 16, DEV, max_requests=4), rng, reqs)
    for got, k in [(whole, "r0"), (cut, "r0")] + [(mixed[k], k) for k in reqs]:
        err = np.abs(got - want[k]).max(-1) / np.abs(want[k]).max()
        assert np.isfinite(got).all() and np.median(err) <= 0.3, (k, float(np.median(err)))
        n = clear[k]
        if n < 8:
            continue
        floor = (np.abs(plain.forward(wide, cfg, reqs[k], round_to=torch.bfloat16).float().numpy() - want[k]).max(-1) / np.abs(want[k]).max())[:n]
        mid, most = 1.5e-2 + 5 * float(np.median(floor)), 3e-2 + 5 * float(np.quantile(floor, 0.85))
        assert np.median(err[:n]) <= mid and np.quantile(err[:n], 0.85) <= most, (k, float(np.median(err[:n])), float(np.quantile(err[:n], 0.85)), mid, most)
