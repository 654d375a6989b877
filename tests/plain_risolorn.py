"""Risolorn, written out plainly in 64-bit: whole sequences, no cache, no batching, one function per mechanism.
It shares nothing with ``ullm_amd``; the GPU tests compare the framework with it.

A model is (config dict as in config.json, {tensor name: 64-bit tensor}).  Linear weights are [out, in].
"""
import math

import torch

F = torch.float64


# ----------------------------------------------------------------------------- small pieces

def dyn_tanh(x, alpha, gain, shift):
    """A squashed stream in place of a normed one: no statistics of the row enter."""
    return torch.tanh(alpha * x) * gain + shift


def normed(x, w, name):
    return dyn_tanh(x, w[name + ".alpha"], w[name], w[name + ".b"])


def over_rms(x, eps):
    """x over its root mean square (eps inside the root), over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit(x):
    """x over its length, over the last axis."""
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def logsigmoid(z):
    return -softplus(-z)


def causal_conv(u, w):
    """u [T, channels], w [channels, taps]: every channel's taps over its own past; the last tap is the token's own input, and
    what lies ahead of the first token counts as zero."""
    T, taps = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for j in range(taps):
        back = taps - 1 - j                                          # how many tokens back column j looks
        if back < T:
            y[back:] += w[:, j] * u[:T - back]
    return y


# ----------------------------------------------------------------------------- gated delta rule

def delta_rule(q, k, v, g, beta):
    """One head: q, k [T, N], v [T, P], g and beta [T].  The memory fades, what it predicts for the key is corrected towards
    the value, and the corrected memory is read."""
    T, P = v.shape
    S = torch.zeros(k.shape[1], P, dtype=v.dtype)
    out = torch.zeros(T, P, dtype=v.dtype)
    for t in range(T):
        S = g[t] * S
        u = beta[t] * (v[t] - k[t] @ S)
        S = S + torch.outer(k[t], u)
        out[t] = q[t] @ S
    return out


def delta_mixer(h, w, p, m, eps):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m.get("vdim", m["dim"])
    q, k, v = (silu(causal_conv(h @ w[f"{p}.{s}"].T, w[f"{p}.{s}.conv"])) for s in "qkv")
    q, k, v = unit(q.view(T, G, d)) * d ** -0.5, unit(k.view(T, G, d)), v.view(T, H, dv)
    beta = torch.sigmoid(h @ w[p + ".b"].T)
    g = torch.exp(-torch.exp(w[p + ".A_log"]) * softplus(h @ w[p + ".a"].T + w[p + ".dt_bias"]))
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for head in range(H):
        kv = head // (H // G)
        out[:, head] = over_rms(delta_rule(q[:, kv], k[:, kv], v[:, head], g[:, head], beta[:, head]), eps) * w[p + ".norm"]
    return (out.reshape(T, H * dv) * silu(h @ w[p + ".g"].T)) @ w[p + ".o"].T


# ----------------------------------------------------------------------------- matrix memory with exponential gates

def exp_gated_memory(q, k, v, i, f):
    """One head: q, k [T, N], v [T, P], log gates i and f [T].  Memory and normaliser are kept over e^m with a running m."""
    T, P = v.shape
    S = torch.zeros(k.shape[1], P, dtype=v.dtype)
    n = torch.zeros(k.shape[1], dtype=v.dtype)
    m = torch.zeros((), dtype=v.dtype)
    out = torch.zeros(T, P, dtype=v.dtype)
    for t in range(T):
        top = torch.maximum(f[t] + m, i[t])
        keep, take = torch.exp(f[t] + m - top), torch.exp(i[t] - top)
        S = keep * S + take * torch.outer(k[t], v[t])
        n = keep * n + take * k[t]
        m = top
        out[t] = (q[t] @ S) / (torch.maximum((n @ q[t]).abs(), torch.exp(-m)) + 1e-6)
    return out


def mlstm_gates(h, w, p, cap):
    soft = lambda z: cap * torch.tanh(z / cap)                       # noqa: E731
    return soft(h @ w[p + ".i"].T + w[p + ".i.b"]), logsigmoid(soft(h @ w[p + ".f"].T + w[p + ".f.b"]))


def mlstm_mixer(h, w, p, m, eps):
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m.get("vdim", m["dim"])
    q = (h @ w[p + ".q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w[p + ".k"].T).view(T, H, d)
    v = (h @ w[p + ".v"].T).view(T, H, dv)
    i, f = mlstm_gates(h, w, p, m["gate_cap"])
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for head in range(H):
        out[:, head] = over_rms(exp_gated_memory(q[:, head], k[:, head], v[:, head], i[:, head], f[:, head]), eps)
    return (out.reshape(T, H * dv) * w[p + ".norm"] * torch.sigmoid(h @ w[p + ".g"].T)) @ w[p + ".o"].T


# ----------------------------------------------------------------------------- attention in chunks with a sink

def rotation(dims, base, scaling):
    """(frequency of every pair, size of the cosines and sines)."""
    freq = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return freq, 1.0
    s, orig = scaling["factor"], scaling["original"]
    at = lambda turns: dims * math.log(orig / (2 * math.pi * turns)) / (2 * math.log(base))      # noqa: E731
    lo, hi = max(math.floor(at(scaling["fast"])), 0), min(math.ceil(at(scaling["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freq):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s * r + f * (1 - r))
    return out, 0.1 * math.log(s) + 1.0


def rotate_adjacent(x, positions, dims, base, scaling):
    """x [T, heads, dim]: dims 2i and 2i+1 of the first ``dims`` turn together."""
    if not dims:
        return x
    freq, size = rotation(dims, base, scaling)
    a = positions.to(F)[:, None] * torch.tensor(freq, dtype=F)[None, :]
    c, s = (a.cos() * size).to(x.dtype)[:, None, :], (a.sin() * size).to(x.dtype)[:, None, :]
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def same_chunk(T, size):
    """[query, key]: keys up to the query itself in the query's own chunk of ``size`` positions (0: all)."""
    i = torch.arange(T)
    seen = i[None, :] <= i[:, None]
    return seen & (i[None, :] // size == i[:, None] // size) if size else seen


def attention(h, w, p, m, eps):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m.get("vdim", m["dim"])
    q = (h @ w[p + ".q"].T + w[p + ".q.b"]).view(T, H, d)
    k = (h @ w[p + ".k"].T + w[p + ".k.b"]).view(T, G, d)
    v = (h @ w[p + ".v"].T + w[p + ".v.b"]).view(T, G, dv)
    rot, at = m.get("rot") or {}, torch.arange(T)
    q = rotate_adjacent(q, at, rot.get("dims", 0), rot.get("base", 1e4), rot.get("scaling"))
    k = rotate_adjacent(k, at, rot.get("dims", 0), rot.get("base", 1e4), rot.get("scaling"))
    seen = same_chunk(T, (m.get("mask") or {}).get("size", 0))
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for head in range(H):
        g = head // (H // G)
        score = ((q[:, head] @ k[:, g].T) * m["scale"]).masked_fill(~seen, -math.inf)
        sink = w[p + ".sink"][head]
        top = torch.maximum(score.max(-1, keepdim=True).values, sink)
        e = torch.exp(score - top)
        out[:, head] = (e @ v[:, g]) / (e.sum(-1, keepdim=True) + torch.exp(sink - top))
    return out.reshape(T, H * dv) @ w[p + ".o"].T


MIXERS = {"delta": delta_mixer, "mlstm": mlstm_mixer, "attention": attention}


# ----------------------------------------------------------------------------- routed feed-forward

MARGINS = None      # a list: every routed layer run appends, per token, how close its choice of groups or experts was


def choose_experts(c, top, groups, keep):
    """(indices of the ``top`` largest of the choice scores ``c`` [n] in the ``keep`` best of ``groups`` equal groups of
    neighbours, a group counting as the sum of its two largest; the smallest gap between what was taken and what was left)."""
    n = c.numel()
    size = n // groups
    worth = torch.sort(c.view(groups, size), descending=True).values[:, :2].sum(-1)
    order = sorted(range(groups), key=lambda g: (-worth[g].item(), g))
    margin = math.inf if keep >= groups else (worth[order[keep - 1]] - worth[order[keep]]).item()
    cand = [e for g in sorted(order[:keep]) for e in range(g * size, (g + 1) * size)]
    cand.sort(key=lambda e: (-c[e].item(), e))
    if top < len(cand):
        margin = min(margin, (c[cand[top - 1]] - c[cand[top]]).item())
    return cand[:top], margin


def routed_ff(h, w, p, f):
    r = f["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    s = torch.sigmoid(h @ w[p + ".router"].T)
    choice = s + w[p + ".correction"]
    out, margins = torch.zeros_like(h), []
    for t in range(h.shape[0]):
        picked, margin = choose_experts(choice[t], r["top"], groups["count"], groups["keep"])
        margins.append(margin)
        for e in picked:
            unit_out = silu(w[f"{p}.e{e}.gate"] @ h[t]) * (w[f"{p}.e{e}.up"] @ h[t])
            out[t] += s[t, e] * (w[f"{p}.e{e}.down"] @ unit_out)
    if MARGINS is not None:
        MARGINS.append(torch.tensor(margins, dtype=F))
    return out


# ----------------------------------------------------------------------------- the model

def forward(w, cfg, tokens, layers_out=None, round_to=None):
    """Logits [T, vocab] of one sequence from its first token; ``layers_out`` receives the stream after every layer.
    With ``round_to`` every sublayer's input is rounded to that dtype on its way (what a model loses at the least when
    its products read such inputs)."""
    rounded = (lambda t: t.to(round_to).to(t.dtype)) if round_to is not None else (lambda t: t)
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(list(tokens))] * (cfg.get("embedding") or {}).get("scale", 1.0)
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}"
        h = rounded(normed(x, w, p + ".norm1"))
        y = MIXERS[L["type"]](h, w, p + ".mix", L["mixer"], eps)
        if L.get("mlp"):
            y = y + routed_ff(h, w, p + ".mlp", L["mlp"])
        x = x + y
        if layers_out is not None:
            layers_out.append(x.clone())
    return rounded(normed(x, w, "final.norm")) @ w["head"].T * cfg.get("logit_scale", 1.0)


# ----------------------------------------------------------------------------- random weights

def tensor_shapes(cfg):
    """{tensor name: shape} of a model of this configuration."""
    W, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, W), "head": (V, W)}

    def norm(name):
        out.update({name: (W,), name + ".b": (W,), name + ".alpha": ()})
    norm("final.norm")
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}", L["mixer"]
        q = p + ".mix"
        norm(p + ".norm1")
        H, d, dv = m["heads"], m["dim"], m.get("vdim", m["dim"])
        G = m.get("kv_heads", H)
        for s, n in (("q", (H if L["type"] != "delta" else G) * d), ("k", G * d), ("v", (G if L["type"] == "attention" else H) * dv)):
            out[f"{q}.{s}"] = (n, W)
            if L["type"] == "delta":
                out[f"{q}.{s}.conv"] = (n, m["conv"])
            if L["type"] == "attention":
                out[f"{q}.{s}.b"] = (n,)
        out[q + ".o"] = (W, H * dv)
        if L["type"] == "attention":
            out[q + ".sink"] = (H,)
        elif L["type"] == "delta":
            out.update({q + ".b": (H, W), q + ".A_log": (H,), q + ".norm": (dv,), q + ".a": (H, W), q + ".dt_bias": (H,),
                        q + ".g": (H * dv, W)})
        else:
            out.update({q + ".g": (H * dv, W), q + ".norm": (H * dv,), q + ".i": (H, W), q + ".i.b": (H,), q + ".f": (H, W),
                        q + ".f.b": (H,)})
        f = L.get("mlp")
        if f:
            n, ff = f["router"]["experts"], f["expert"]["ff"]
            out.update({p + ".mlp.router": (n, W), p + ".mlp.correction": (n,)})
            for e in range(n):
                out.update({f"{p}.mlp.e{e}.gate": (ff, W), f"{p}.mlp.e{e}.up": (ff, W), f"{p}.mlp.e{e}.down": (W, ff)})
    return out


def random_weights(cfg, seed):
    """bfloat16 tensors of a model of this configuration, sized so that every mechanism matters in the logits."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last, W = name.rsplit(".", 1)[-1], cfg["width"]
        r = torch.randn(shape, generator=g)
        if last == "alpha":
            t = 0.7 + 0.2 * r
        elif last in ("norm1", "norm") and len(shape) == 1:
            t = 1.0 + 0.2 * r
        elif last == "conv":
            t = r / math.sqrt(shape[-1])
        elif name.endswith(".f.b"):
            t = 3.0 + 1.5 * r                                        # memories of tens of tokens
        elif last == "b" and len(shape) == 1:
            t = 0.3 * r
        elif last == "sink":
            t = 0.5 + r
        elif last == "A_log":
            t = torch.log(torch.rand(shape, generator=g) * 2 + 0.05)
        elif last == "dt_bias":
            t = -3.0 + 1.5 * r
        elif last == "correction":
            t = 0.3 * r
        elif last == "embed":
            t = r
        else:
            t = r * 1.2 / math.sqrt(shape[-1])
        out[name] = t.to(torch.bfloat16)
    return out


def greedy_generate(w, cfg, prompt, n):
    """The n tokens that follow ``prompt`` when the largest logit is taken every time (the lowest index on a tie)."""
    toks, out = list(prompt), []
    for _ in range(n):
        nxt = int(torch.argmax(forward(w, cfg, toks)[-1]))
        toks.append(nxt)
        out.append(nxt)
    return out
