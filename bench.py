#!/usr/bin/env python3
"""Decode and prefill throughput of the engine at Qwen3 layer sizes with random weights.

    python bench.py --gpus 1 --steps K --warmup W

One JSON line.  ``value`` = decoded tokens per second at batch 8 of Qwen3-8B sizes (every request with a
1024-token prompt), timed over exactly K engine steps (schedule + model step + sampling) after W untimed
ones.  ``prefill`` = one 2048-token prompt.  ``roofline`` = bytes a decode step has to read (every weight
once + the live requests' cache) over its time, against 8 TB/s (``frac``) and against what a kernel that
only reads reaches on this GPU (``frac_of_measured``).  ``points`` = tokens per second of the other workloads
(decode at batch 1 and 64; batch 8 at 16K-token, batch 64 at 8K-token and batch 1 at 32K-token contexts; a
16,384-token prompt; Qwen3-14B and Qwen3-32B sizes at batch 8, Qwen3-32B at batch 64 with 4096-token contexts
and its 2048-token prefill; the 256-request mixed workloads at Qwen3-14B and Qwen3-0.6B sizes);
``points_detail`` says at which context each ran and how far from its roofline.  ``measured_peaks`` = a
streaming read, a device copy and a large bfloat16 product on this GPU.  The reference publishes no number for this configuration, so ``vs_baseline`` is null.
"""
import argparse
import json
import os
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, ROOT)

HBM_PEAK_GBS = 8000.0
PEAK_FLOPS = {"bfloat16": 2.5e15, "float32": 157.3e12}
# the reference's own benchmark (bench.py:10-45, README.md:129-147): Qwen3-0.6B, 256 requests, prompt and
# generation lengths uniform in 100..1024, temperature 0.6, no end-of-sequence; 9032.37 tokens/s on an A100 40GB
REFERENCE_MIXED_TOK_S = 9032.37
SIZES = ("0.6b", "8b", "14b", "32b")
LONGEST_CONTEXT = 32768 + 64       # the longest context any point of the default run reaches


def parse_args():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=64)
    ap.add_argument("--warmup", type=int, default=8)
    ap.add_argument("--layers", type=int, default=None, help="run fewer layers than the configuration has")
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--prompt-len", type=int, default=1024)
    ap.add_argument("--context-len", type=int, default=4096)
    ap.add_argument("--dtype", default="bfloat16")
    ap.add_argument("--top-k", type=int, default=-1, help="top-k of the decode requests (default: off)")
    ap.add_argument("--top-p", type=float, default=1.0, help="top-p of the decode requests (default: off)")
    ap.add_argument("--no-points", action="store_true", help="only the headline decode point")
    ap.add_argument("--eager", action="store_true", help="no HIP graphs")
    ap.add_argument("--size", choices=SIZES, default=None,
                    help="layer sizes of this Qwen3 model (default 8b; 0.6b for --mixed-only)")
    ap.add_argument("--mixed-only", action="store_true",
                    help="only the reference's own workload: 256 requests of mixed lengths "
                         "(Qwen3-0.6B sizes unless --size is given)")
    ap.add_argument("--design", choices=sorted(DESIGN_SHAPES), default=None, metavar="SHAPE",
                    help="instead of the default workload: Pamopel (attention with a distance bias and head gates, a "
                         "layer on another's keys and values, a Mamba-2 layer) beside a Qwen3 stack of the same width, "
                         f"heads, feed-forward, vocabulary and depth, random weights; shapes: {sorted(DESIGN_SHAPES)}")
    ap.add_argument("--design-model", choices=("both", "all", "pamopel", "qwen3", "ziferax", "dovisun", "kumudra", "nadevik", "risolorn"), default="both",
                    help="with --design: one design only (for profiles), Pamopel and Qwen3 (both), or these, Ziferax "
                         "(a stack of parallel blocks of windowed attention with sinks and a routed feed-forward) and "
                         "Dovisun (parallel blocks of unit-norm attention with a fixed sink or latent attention, dense "
                         "or routed feed-forwards, two layers passed twice) and Kumudra (two copies of the residual "
                         "stream, gated linear attention, lightning attention and windowed attention beside time "
                         "mixing, four layers passed twice) and Nadevik (norms behind the sublayers, sigmoid attention "
                         "over a window and pooled blocks beside a selective scan, windowed latent attention, experts "
                         "from the best groups) and Risolorn (parallel blocks behind a dynamic tanh: the gated delta "
                         "rule, a matrix memory with exponential gates, attention in chunks with sinks) (all)")
    ap.add_argument("--prefill-only", type=int, default=0, metavar="T",
                    help="only time a T-token prompt and print its figures (for profiling)")
    return ap.parse_args()


def weight_bytes(model, itemsize):
    """Bytes of every weight a decode step reads once (the embedding table is only gathered)."""
    total = 0
    for d in model.weight_decls():
        if d.name == model.plan.embedding_weight and not model.plan.tie_head_to_embedding:
            continue
        n = 1
        for s in d.shape:
            n *= s
        total += n * (4 if d.keep_fp32 else itemsize)
    return total


def step_flops(cfg, n_tokens, kv_lens_sum_causal, n_logit_rows):
    """Multiply-adds * 2 of one step: projections per token, attention scores and values, head."""
    H, nq, nkv, hd, I, L, V = (cfg.hidden_size, cfg.num_attention_heads, cfg.num_key_value_heads, cfg.head_dim,
                               cfg.intermediate_size, cfg.num_hidden_layers, cfg.vocab_size)
    per_token = 2 * (H * (nq + 2 * nkv) * hd + nq * hd * H + 3 * H * I)
    attn = 4 * nq * hd * kv_lens_sum_causal
    return L * (per_token * n_tokens + attn) + 2 * H * V * n_logit_rows


def measured_peaks():
    """What this GPU reaches with a kernel that only reads (4 GiB, non-temporal 16-byte loads: what a decode
    step's weight streaming could reach at best), on a plain device-to-device copy (bytes read + written per
    second) and on a large square bfloat16 product of the library: the practical ceilings beside the datasheet's."""
    import torch
    from ullm_amd.kernels import ops
    src = torch.empty(1 << 30, dtype=torch.float32, device="cuda:0").normal_()
    for _ in range(2):
        ops.stream_read(src)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(5):
        ops.stream_read(src)
    torch.cuda.synchronize()
    read_gbs = 5 * src.numel() * 4 / (time.perf_counter() - t0) / 1e9
    dst = torch.empty_like(src)
    for _ in range(2):
        dst.copy_(src)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(5):
        dst.copy_(src)
    torch.cuda.synchronize()
    copy_gbs = 5 * 2 * src.numel() * 4 / (time.perf_counter() - t0) / 1e9
    del src, dst
    n = 8192
    a = torch.randn(n, n, device="cuda:0", dtype=torch.bfloat16)
    b = torch.randn(n, n, device="cuda:0", dtype=torch.bfloat16)
    for _ in range(3):
        torch.mm(a, b)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(10):
        torch.mm(a, b)
    torch.cuda.synchronize()
    gemm_tflops = 10 * 2 * n ** 3 / (time.perf_counter() - t0) / 1e12
    del a, b
    torch.cuda.empty_cache()
    return {"read_GBs": round(read_gbs, 1), "copy_GBs": round(copy_gbs, 1), "gemm_bf16_8192_TFLOPs": round(gemm_tflops, 1)}


# Layer shapes for --design: (width, query heads, kv heads, head size, feed-forward, layers) and the
# state-space layer's (heads, head size, state, groups).  Vocabulary 32 768 for both designs.
DESIGN_SHAPES = {"2048": ((2048, 16, 8, 128, 6144, 8), (64, 64, 128, 8)),
                 "4096": ((4096, 32, 8, 128, 12288, 8), (128, 64, 128, 8))}
DESIGN_VOCAB = 32768


def design_configs(shape):
    """(Pamopel config.json, Qwen3 config.json) of one shape: Pamopel's layers repeat attention, attention on the
    layer before's keys and values, Mamba-2, attention; every layer has the feed-forward."""
    (W, H, G, D, F, L), (mh, mp, mn, mg) = DESIGN_SHAPES[shape]
    att = dict(heads=H, kv_heads=G, dim=D, vdim=D, scale=D ** -0.5, bias_max=1024)
    mlp = dict(kind="dense", ff=F)
    layers = []
    for i in range(L):
        kind = i % 4
        if kind == 2:
            layers.append(dict(type="mamba2", mlp=mlp, mixer=dict(heads=mh, vdim=mp, state=mn, groups=mg, conv=4, norm_groups=mg)))
        else:
            layers.append(dict(type="attention", mlp=mlp, mixer=dict(att, kv_from=i - 1) if kind == 1 else dict(att)))
    pamopel = dict(architecture="Pamopel", vocab=DESIGN_VOCAB, width=W, layers=layers, norm=dict(eps=1e-5), residual_mult=0.5,
                   logit_scale=1.0, embedding=dict(scale=1.0, bigram=dict(buckets=65521, mul_prev=8191, mul_cur=127)))
    qwen = dict(architectures=["Qwen3ForCausalLM"], hidden_size=W, num_hidden_layers=L, num_attention_heads=H,
                num_key_value_heads=G, head_dim=D, intermediate_size=F, vocab_size=DESIGN_VOCAB, rope_theta=1e6,
                rms_norm_eps=1e-6, max_position_embeddings=40960, tie_word_embeddings=False, attention_bias=False,
                use_sliding_window=False, initializer_range=0.02, torch_dtype="bfloat16")
    return pamopel, qwen


# Ziferax at a design shape: the same width, heads and depth; a window of 1024 keys, half of each head rotated; per
# token as many feed-forward columns as the dense stack has (top 4 of 32 experts of a sixth of it each, four identity
# experts beside them, and a shared expert of a third of it), so a token's products are of equal size.
def ziferax_config(shape):
    (W, H, G, D, F, L), _ = DESIGN_SHAPES[shape]
    mixer = dict(heads=H, kv_heads=G, dim=D, vdim=D, scale=D ** -0.5, mask=dict(size=1024), rot=dict(base=500000.0, dims=D // 2))
    mlp = dict(kind="moe", router=dict(experts=32, identity=4, top=4), expert=dict(ff=F // 6, limit=7.0),
               shared=dict(ff=F // 3, limit=7.0))
    return dict(architecture="Ziferax", vocab=DESIGN_VOCAB, width=W, norm=dict(eps=1e-5), residual_mult=0.5,
                layers=[dict(type="attention", mixer=mixer, mlp=mlp) for _ in range(L)])


# Dovisun at a design shape: the same width and heads; six layers of which the third and fourth are passed twice, so
# eight layer runs a token as the other stacks have; attention layers without positions (unit-norm queries and keys, a
# fixed sink) and one latent-attention layer in four (a kv latent of 192 and 64 rotated dims: 256 cached values a
# token, the largest head the matrix-core attention kernels take, against 2 * 8 * 128 of an attention layer; a q
# latent of 3/8 of the width); dense feed-forwards of the dense
# stack's size without a gate, and routed ones of as many columns a token (top 4 of 32 experts of a sixth of it).
def dovisun_config(shape):
    (W, H, G, D, F, L), _ = DESIGN_SHAPES[shape]
    att = dict(heads=H, kv_heads=G, dim=D, vdim=D, scale=D ** -0.5)
    latent = dict(heads=H, dim=D, rot_dim=D // 2, vdim=D, q_rank=W * 3 // 8, kv_rank=192, scale=(D + D // 2) ** -0.5,
                  rot=dict(base=1e6, dims=D // 2, scaling=dict(factor=8.0, original=4096, fast=32.0, slow=1.0)))
    dense = dict(kind="dense", ff=F)
    moe = dict(kind="moe", router=dict(experts=32, top=4), expert=dict(ff=F // 6))
    layers = [dict(type="attention", mixer=att, mlp=dense), dict(type="attention", mixer=att, mlp=moe),
              dict(type="latent_attention", mixer=latent, mlp=dense), dict(type="attention", mixer=att, mlp=moe),
              dict(type="attention", mixer=att, mlp=dense), dict(type="attention", mixer=att, mlp=moe)]
    return dict(architecture="Dovisun", vocab=DESIGN_VOCAB, width=W, norm=dict(eps=1e-5), layers=layers[:max(4, L - 2)],
                embedding=dict(scale=float(W) ** 0.5), logit_softcap=30.0, loop=dict(start=2, stop=4, times=2))


# Kumudra at a design shape: the same width; four layers passed twice, so eight layer runs a token as the other stacks
# have, over two copies of the residual stream: two lightning layers, gated linear attention (keys of half the head
# size) with the dense feed-forward, and one layer of windowed attention (the other stacks' heads, a window of 1024 keys,
# half of each head rotated) beside time mixing (heads of 64), these three with routed feed-forwards of as many columns
# a token as the dense one (top 4 of 32 experts of a sixth of it).
def kumudra_config(shape):
    (W, H, G, D, F, L), _ = DESIGN_SHAPES[shape]
    moe = dict(kind="moe", router=dict(experts=32, top=4, scale=2.5), expert=dict(ff=F // 6))
    gla = dict(type="gla", mixer=dict(heads=H, dim=D // 2, vdim=D, tau=8.0), mlp=dict(kind="dense", ff=F))
    lightning = dict(heads=H, dim=D, vdim=D, decay=[1.0 - 2.0 ** (-5.0 - 4.0 * h / max(1, H - 1)) for h in range(H)])
    left = dict(heads=H, kv_heads=G, dim=D, vdim=D, scale=D ** -0.5, mask=dict(size=1024),
                rot=dict(base=500000.0, dims=D // 2, scaling=dict(factor=4.0, low=1.0, high=8.0, original=8192)))
    layers = [dict(type="lightning", mixer=lightning, mlp=moe), gla,
              dict(type="parallel", mlp=moe, mixer=dict(left=left, right=dict(heads=W // 64, dim=64), left_scale=0.5, right_scale=1.0)),
              dict(type="lightning", mixer=lightning, mlp=moe)]
    return dict(architecture="Kumudra", vocab=DESIGN_VOCAB, width=W, norm=dict(eps=1e-5), layers=layers, streams=2,
                residual_mult=0.5, embedding=dict(scale=1.0), loop=dict(start=0, stop=4, times=max(1, L // 4)))


# Nadevik at a design shape: the same width, heads and depth.  Of every four layers the first and the last are two mixers
# side by side, attention (the other stacks' heads, a window of 1024 keys, beyond it a key per block of 16 tokens) and a
# selective scan (twice the width, 16 states a channel, step sizes of rank width / 16); the second is latent attention (the
# other latent stack's sizes, the same window) and the third reads the second's latents.  Every feed-forward is routed,
# with as many columns a token as the dense stack's (top 4 of 32 experts of a sixth of it, in four groups of which three
# are kept).
def nadevik_config(shape):
    (W, H, G, D, F, L), _ = DESIGN_SHAPES[shape]
    mlp = dict(kind="moe", router=dict(experts=32, top=4, groups=dict(count=4, keep=3)), expert=dict(ff=F // 6, limit=7.0))
    left = dict(heads=H, kv_heads=G, dim=D, vdim=D, conv=4, scale=D ** -0.5, softcap=30.0, mask=dict(size=1024, pool=16))
    parallel = dict(left=left, right=dict(inner=2 * W, state=16, dt_rank=W // 16, conv=4), left_scale=0.7, right_scale=0.8)
    latent = dict(heads=H, dim=D, rot_dim=D // 2, vdim=D, kv_rank=192, scale=(D + D // 2) ** -0.5, mask=dict(size=1024),
                  rot=dict(base=1e6, dims=D // 2))
    layers = []
    for i in range(L):
        if i % 4 in (0, 3):
            layers.append(dict(type="parallel", mixer=parallel, mlp=mlp))
        else:
            layers.append(dict(type="latent_attention", mixer=dict(latent, kv_from=i - 1) if i % 4 == 2 else latent, mlp=mlp))
    return dict(architecture="Nadevik", vocab=DESIGN_VOCAB, width=W, norm=dict(eps=1e-6), canon=dict(taps=4), layers=layers,
                embedding=dict(scale=float(W) ** 0.5, bigram=dict(buckets=65521, mul_prev=8191, mul_cur=127)))


# Risolorn at a design shape: the same width, heads and depth.  Of every four layers one is a matrix memory with exponential
# gates and two are the gated delta rule (heads of the head size, as many states as Kumudra's lightning layers have; the
# other stacks' key heads, four taps), one attention (the other stacks' heads, chunks of 2048 positions, sinks, half of each
# head rotated, stretched).  Every feed-forward is routed, with as many columns a token as the dense stack's (top 4 of 32
# experts of a sixth of it, in four groups of which three are kept).
def risolorn_config(shape):
    (W, H, G, D, F, L), _ = DESIGN_SHAPES[shape]
    mlp = dict(kind="moe", router=dict(experts=32, top=4, groups=dict(count=4, keep=3)), expert=dict(ff=F // 6))
    delta = dict(type="delta", mlp=mlp, mixer=dict(heads=H, kv_heads=G, dim=D, vdim=D, conv=4))
    memory = dict(type="mlstm", mlp=mlp, mixer=dict(heads=H, dim=D, vdim=D, gate_cap=10.0))
    rot = dict(base=500000.0, dims=D // 2, scaling=dict(factor=8.0, original=4096, fast=32.0, slow=1.0))
    att = dict(type="attention", mlp=mlp, mixer=dict(heads=H, kv_heads=G, dim=D, vdim=D, scale=D ** -0.5, mask=dict(size=2048), rot=rot))
    return dict(architecture="Risolorn", vocab=DESIGN_VOCAB, width=W, norm=dict(eps=1e-6), embedding=dict(scale=1.0), logit_scale=0.7,
                layers=[(memory, delta, att, delta)[i % 4] for i in range(L)])


def design_run(args):
    """Decode at batch 1 / 8 / 64 (1024-token prompts) and one 2048-token prompt, for the designs of a shape."""
    out = {"metric": f"decode and prefill tok/s, designs beside Qwen3 at shape {args.design}, random weights",
           "unit": "tokens/s", "dtype": args.dtype, "data": "synthetic", "shape": args.design, "designs": {}}
    configs = design_configs(args.design) + (ziferax_config(args.design), dovisun_config(args.design), kumudra_config(args.design),
                                             nadevik_config(args.design), risolorn_config(args.design))
    for label, config in zip(("pamopel", "qwen3", "ziferax", "dovisun", "kumudra", "nadevik", "risolorn"), configs):
        if args.design_model not in ("both", "all", label) or (label not in ("pamopel", "qwen3") and args.design_model == "both"):
            continue
        m = Sized(label, args.dtype, 4096, eager=args.eager, config=config)
        rec = {"weights_GB": round(m.wbytes / 1e9, 3), "decode": {}}
        # for profiles: --prefill-only T times the prompt alone, --no-points the decode steps at --batch alone
        for batch in () if args.prefill_only else (args.batch,) if args.no_points else (1, 8, 64):
            tok_s, ms, _, ctx = m.decode(batch, args.steps, args.warmup, 1024)
            rec["decode"][f"b{batch}"] = {"tok_s": round(tok_s, 1), "ms_per_step": round(ms, 3), "context": round(ctx)}
        if not args.no_points or args.prefill_only:
            n = args.prefill_only or 2048
            p_tok_s, p_ms, _ = m.prefill(n)
            rec[f"prefill_{n}"] = {"tok_s": round(p_tok_s, 1), "ms": round(p_ms, 3)}
        out["designs"][label] = rec
        m.close()
    print(json.dumps(out))
    return 0


class Sized:
    """A model of one named size with random weights on the device, and the runs it is timed on."""

    def __init__(self, size, dtype, context_len, layers=None, eager=False, longest_context=None, config=None):
        """``config``: a config.json dict of any registered architecture instead of a named Qwen3 size
        (``size`` is then only its label)."""
        import torch
        from ullm_amd.config import parse_random_weights
        from ullm_amd.engine.loading import make_env
        from ullm_amd.models import build_model
        from ullm_amd.weights.random_init import bind_random_weights
        self.torch, self.size, self.dtype, self.context_len, self.eager = torch, size, dtype, context_len, eager
        if config is None:
            config, _ = parse_random_weights(f"qwen3-{size}")
            self.full_layers = config["num_hidden_layers"]
            if layers is not None:
                config["num_hidden_layers"] = layers
        self.cfg, self.model = build_model(config)
        # the model (its position table) is built once for the longest context any point runs at; every engine
        # gets an environment with its own context length (block tables as wide as that context needs)
        self.env = make_env(dtype, "cuda:0", max(context_len, longest_context or 0))
        bind_random_weights(self.model, self.env, seed=0)
        self.itemsize = 2 if dtype == "bfloat16" else 4
        self.wbytes = weight_bytes(self.model, self.itemsize)
        self.kv_per_token = sum(g.bytes_per_token(self.itemsize) for g in self.model.cache_layout()[0])
        self.gen = torch.Generator().manual_seed(0)

    def engine(self, context_len=None, **kw):
        import dataclasses
        from ullm_amd import EngineConfig
        from ullm_amd.engine.engine import Engine
        context_len = context_len or self.context_len
        ec = EngineConfig(model="(random weights)", dtype=self.dtype, context_len=context_len, page_size=16,
                          enforce_eager=self.eager, **kw)
        return Engine(ec, model=self.model, env=dataclasses.replace(self.env, context_len=context_len), model_config=self.cfg)

    def _check_finite_once(self, eng):
        """The next step's logits must be finite (checked outside the timed steps)."""
        torch = self.torch

        def check(sampling, logits):
            eng.on_logits = None
            if not bool(torch.isfinite(logits).all()):
                raise RuntimeError(f"Qwen3-{self.size}: a step returned logits that are not finite")
        eng.on_logits = check

    def decode(self, batch, steps, warmup, prompt_len, top_k=-1, top_p=1.0, context_len=None):
        """(tokens/s, ms per step, bytes read per step, mean context) over exactly ``steps`` engine steps."""
        from ullm_amd import SamplingParams
        torch = self.torch
        budget = max(8192, batch)
        # requests that finish their prompt early decode while the others are still in theirs
        new_tokens = warmup + steps + 4 + -(-batch * prompt_len // budget)
        eng = self.engine(context_len=context_len, max_bs=batch, num_pages=batch * (-(-(prompt_len + new_tokens + 16) // 16)),
                          max_num_batched_tokens=budget, max_prefill_chunk=2048)
        for i in range(batch):
            prompt = torch.randint(0, self.cfg.vocab_size, (prompt_len,), generator=self.gen).tolist()
            eng.add_request(f"r{i}", prompt, SamplingParams(temperature=0.6, top_k=top_k, top_p=top_p, ignore_eos=True,
                                                            seed=i, max_new_tokens=new_tokens))
        while any(r.num_computed < prompt_len for r in eng.scheduler.requests.values()) or eng.scheduler.waiting:
            eng.step()                                   # prefill (untimed)
        self._check_finite_once(eng)
        for _ in range(max(1, warmup)):
            eng.step()
        ctx_before = sum(r.num_tokens for r in eng.scheduler.requests.values())
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        for _ in range(steps):
            out = eng.step()
            assert len(out) == batch
        torch.cuda.synchronize()
        dt = time.perf_counter() - t0
        ctx_after = sum(r.num_tokens for r in eng.scheduler.requests.values())
        mean_ctx = (ctx_before + ctx_after) / 2.0
        for rid in list(eng.scheduler.requests):
            eng.abort_request(rid)
        del eng
        torch.cuda.empty_cache()
        return batch * steps / dt, dt / steps * 1e3, self.wbytes + self.kv_per_token * mean_ctx, mean_ctx / batch

    def prefill(self, n_tokens):
        """(tokens/s, ms, fraction of the dtype's matrix peak) of one prompt of n_tokens, best of three."""
        from ullm_amd import SamplingParams
        torch = self.torch
        context_len = max(self.context_len, n_tokens + 16)
        if context_len > self.env.context_len:
            # the engine would keep the prompt's last context_len tokens and the figures would be of those
            raise SystemExit(f"a prompt of {n_tokens} tokens needs --context-len above {n_tokens} (it is {self.context_len})")
        eng = self.engine(context_len=context_len, max_bs=1, num_pages=-(-(n_tokens + 16) // 16),
                          max_num_batched_tokens=n_tokens, max_prefill_chunk=n_tokens)
        best = None
        for rep in range(4):
            prompt = torch.randint(0, self.cfg.vocab_size, (n_tokens,), generator=self.gen).tolist()
            eng.add_request(f"p{rep}", prompt, SamplingParams(temperature=0.0, max_new_tokens=1, ignore_eos=True))
            if rep == 0:
                self._check_finite_once(eng)
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            out = eng.step()
            torch.cuda.synchronize()
            dt = time.perf_counter() - t0
            assert len(out) == 1 and out[0].is_finished
            if rep > 0:
                best = dt if best is None else min(best, dt)
        del eng
        torch.cuda.empty_cache()
        if not hasattr(self.cfg, "num_attention_heads"):
            return n_tokens / best, best * 1e3, None        # no flop count for this architecture
        flops = step_flops(self.cfg, n_tokens, n_tokens * (n_tokens + 1) // 2, 1)
        return n_tokens / best, best * 1e3, flops / best / PEAK_FLOPS[self.dtype]

    def mixed(self):
        """Output tokens per second over 256 requests arriving at once (prompt and generation lengths uniform
        in 100..1024, temperature 0.6, no end-of-sequence), continuous batching; returns (tokens/s, output
        tokens, seconds, engine steps)."""
        import random
        from ullm_amd import SamplingParams
        torch = self.torch
        rng = random.Random(0)
        n = 256
        prompts = [[rng.randint(0, 10000) for _ in range(rng.randint(100, 1024))] for _ in range(n)]
        new_tokens = [rng.randint(100, 1024) for _ in range(n)]
        eng = self.engine(max_bs=256, num_pages=n * 130, max_num_batched_tokens=8192, max_prefill_chunk=2048)
        eng.add_request("warm", prompts[0][:64], SamplingParams(temperature=0.6, ignore_eos=True, max_new_tokens=10))
        self._check_finite_once(eng)
        while eng.has_unfinished_requests():
            eng.step()
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        for i in range(n):
            eng.add_request(f"m{i}", prompts[i], SamplingParams(temperature=0.6, ignore_eos=True, seed=i,
                                                                max_new_tokens=new_tokens[i]))
        steps = 0
        while eng.has_unfinished_requests():
            eng.step()
            steps += 1
        torch.cuda.synchronize()
        dt = time.perf_counter() - t0
        del eng
        torch.cuda.empty_cache()
        return sum(new_tokens) / dt, sum(new_tokens), dt, steps

    def close(self):
        del self.model
        self.torch.cuda.empty_cache()


def decode_detail(tok_s, ms, bytes_step, ctx, read_gbs):
    achieved = bytes_step / (ms * 1e-3) / 1e9
    return {"tok_s": round(tok_s, 2), "ms_per_step": round(ms, 4), "context": round(ctx, 1),
            "GBs": round(achieved, 1), "frac": round(achieved / HBM_PEAK_GBS, 4),
            "frac_of_measured": round(achieved / read_gbs, 4) if read_gbs else None}


def main():
    args = parse_args()
    if args.gpus != 1:
        print(f"bench.py: this engine runs on one GPU; --gpus {args.gpus} is not supported")
        return 2
    if args.design:
        return design_run(args)
    if args.mixed_only:
        size = args.size or "0.6b"
        m = Sized(size, args.dtype, 4096, eager=args.eager)
        tok_s, n_out, secs, steps = m.mixed()
        print(json.dumps({"metric": f"output tok/s, 256 requests, lengths 100..1024 in and out, Qwen3-{size} sizes",
                          "value": round(tok_s, 1), "unit": "tokens/s", "output_tokens": n_out,
                          "seconds": round(secs, 3), "engine_steps": steps,
                          "vs_baseline": round(tok_s / REFERENCE_MIXED_TOK_S, 3) if size == "0.6b" else None,
                          "baseline": "9032.37 tokens/s, the reference with Qwen3-0.6B on an A100 40GB"}))
        return 0
    args.size = args.size or "8b"
    long_points = not args.no_points and not args.prefill_only
    m = Sized(args.size, args.dtype, args.context_len, args.layers, args.eager,
              longest_context=LONGEST_CONTEXT if long_points else args.prefill_only + 16)
    cfg = m.cfg
    if args.prefill_only:
        p_tok_s, p_ms, p_frac = m.prefill(args.prefill_only)
        print(json.dumps({"prefill": {"value": round(p_tok_s, 1), "tokens": args.prefill_only, "ms": round(p_ms, 3),
                                      "frac": round(p_frac, 4)}}))
        return 0
    peaks = measured_peaks() if not args.no_points else {}
    copy_gbs = peaks.get("read_GBs")        # the denominator of frac_of_measured: a kernel that only reads
    tok_s, ms, bytes_step, ctx = m.decode(args.batch, args.steps, args.warmup, args.prompt_len, args.top_k, args.top_p)
    head = decode_detail(tok_s, ms, bytes_step, ctx, copy_gbs)
    line = {
        "metric": f"decode tok/s at bs {args.batch} (also bs 1/64, prefill tok/s at 2048; % of roofline), Qwen3-{args.size}",
        "value": round(tok_s, 2), "unit": "tokens/s", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": round(ms, 4), "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "dtype": "bf16" if args.dtype == "bfloat16" else "fp32", "data": "synthetic",
        "config": {"model": f"Qwen3-{args.size} sizes, random weights", "layers": cfg.num_hidden_layers,
                   "layers_of_config": m.full_layers, "hidden_size": cfg.hidden_size,
                   "num_attention_heads": cfg.num_attention_heads, "num_key_value_heads": cfg.num_key_value_heads,
                   "head_dim": cfg.head_dim, "intermediate_size": cfg.intermediate_size, "vocab_size": cfg.vocab_size,
                   "global_batch": args.batch, "prompt_len": args.prompt_len, "seq_len": args.context_len,
                   "context_at_timing": head["context"], "page_size": 16,
                   "sampling": "temperature 0.6, seeded" + (f", top-k {args.top_k}" if args.top_k > 0 else "") + (f", top-p {args.top_p}" if args.top_p < 1 else ""),
                   "parallelism": "single GPU", "hip_graphs": not args.eager},
        "roofline": {"bound": "hbm", "achieved": head["GBs"], "peak": HBM_PEAK_GBS, "unit": "GB/s", "frac": head["frac"],
                     "frac_of_measured": head["frac_of_measured"]},
    }
    if not args.no_points:
        line["measured_peaks"] = peaks
        p_tok_s, p_ms, p_frac = m.prefill(2048)
        line["prefill"] = {"value": round(p_tok_s, 1), "tokens": 2048, "ms": round(p_ms, 3), "frac": round(p_frac, 4)}
        if peaks.get("gemm_bf16_8192_TFLOPs") and args.dtype == "bfloat16":
            line["prefill"]["frac_of_measured"] = round(p_frac * PEAK_FLOPS["bfloat16"] / (peaks["gemm_bf16_8192_TFLOPs"] * 1e12), 4)
        detail = {}
        b1 = m.decode(1, min(args.steps, 32), min(args.warmup, 4), args.prompt_len)
        b64 = m.decode(64, min(args.steps, 32), min(args.warmup, 4), args.prompt_len)
        # the same batch with the sampling of Qwen3's generation_config.json (top-k 20, top-p 0.95)
        b8f = m.decode(args.batch, args.steps, args.warmup, args.prompt_len, top_k=20, top_p=0.95)
        detail["decode_b1"] = decode_detail(*b1, copy_gbs)
        detail["decode_b64"] = decode_detail(*b64, copy_gbs)
        points = {"decode_b1": round(b1[0], 2), "decode_b64": round(b64[0], 2),
                  f"decode_b{args.batch}_top_k20_top_p95": round(b8f[0], 2)}
        if args.size == "8b" and args.dtype == "bfloat16":
            # further contexts: where the cache outweighs the weights
            for name, batch, ctx in (("decode_b8_ctx16k", 8, 16384), ("decode_b64_ctx8k", 64, 8192), ("decode_b1_ctx32k", 1, 32768)):
                d = m.decode(batch, 16, 2, ctx - 128, context_len=ctx + 64)
                detail[name] = decode_detail(*d, copy_gbs)
                points[name] = round(d[0], 2)
            p16 = m.prefill(16384)
            points["prefill_16384"] = round(p16[0], 1)
            detail["prefill_16384"] = {"tok_s": round(p16[0], 1), "ms": round(p16[1], 3), "frac": round(p16[2], 4)}
        m.close()
        if args.size == "8b" and args.layers is None and args.dtype == "bfloat16":
            # Qwen3-32B sizes: batch 64 with 4096-token contexts (about 69 GB of cache) and a 2048-token prompt
            big = Sized("32b", args.dtype, 4096 + 64, eager=args.eager)
            d32 = big.decode(64, 16, 2, 4096 - 32)
            detail["decode_32b_b64_ctx4096"] = decode_detail(*d32, copy_gbs)
            points["decode_32b_b64_ctx4096"] = round(d32[0], 2)
            d32 = big.decode(8, 16, 2, 1024)
            detail["decode_32b_b8"] = decode_detail(*d32, copy_gbs)
            points["decode_32b_b8"] = round(d32[0], 2)
            p32 = big.prefill(2048)
            points["prefill_32b_2048"] = round(p32[0], 1)
            detail["prefill_32b_2048"] = {"tok_s": round(p32[0], 1), "ms": round(p32[1], 3), "frac": round(p32[2], 4)}
            big.close()
            # the 256-request workload at Qwen3-14B sizes, and the reference's own at Qwen3-0.6B sizes
            mid = Sized("14b", args.dtype, 4096, eager=args.eager)
            d14 = mid.decode(8, 16, 2, 1024)
            detail["decode_14b_b8"] = decode_detail(*d14, copy_gbs)
            points["decode_14b_b8"] = round(d14[0], 2)
            m14 = mid.mixed()
            points["mixed_qwen3_14b"] = round(m14[0], 1)
            detail["mixed_qwen3_14b"] = {"output_tok_s": round(m14[0], 1), "output_tokens": m14[1],
                                         "seconds": round(m14[2], 3), "engine_steps": m14[3]}
            mid.close()
        small = Sized("0.6b", args.dtype, 4096, eager=args.eager)
        m_tok_s, m_out, m_secs, _ = small.mixed()
        small.close()
        points["mixed_qwen3_0p6b"] = round(m_tok_s, 1)
        line["points"] = points
        line["points_detail"] = detail
        # the reference's own benchmark (Qwen3-0.6B, 256 requests); its 9032.37 tokens/s are from an A100 40GB
        line["mixed_qwen3_0p6b"] = {"value": round(m_tok_s, 1), "unit": "output tokens/s", "output_tokens": m_out,
                                    "seconds": round(m_secs, 3),
                                    "vs_reference_a100": round(m_tok_s / REFERENCE_MIXED_TOK_S, 3)}
    print(json.dumps(line))
    return 0


if __name__ == "__main__":
    sys.exit(main())
