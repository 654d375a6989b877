"""Nadevik, written out plainly in 64-bit: whole sequences, no cache, no batching, one function per mechanism.
It shares nothing with ``ullm_amd``; the GPU tests compare the framework with it.

A model is (config dict as in config.json, {tensor name: 64-bit tensor}).  Linear weights are [out, in].
"""
import math

import torch

F = torch.float64


# ----------------------------------------------------------------------------- small pieces

def rms_norm(x, gain, eps):
    """x over its root mean square (eps inside the root), over the last axis, times ``gain``."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * gain


def silu(z):
    return z * torch.sigmoid(z)


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


def rotate_adjacent(x, positions, dims, base):
    """x [T, heads, dim]: dims 2i and 2i+1 of the first ``dims`` turn by position * base^(-2i/dims)."""
    half = dims // 2
    if half == 0:
        return x
    f = torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(half)], dtype=F)
    a = positions.to(F)[:, None] * f[None, :]
    c, s = a.cos()[:, None, :], a.sin()[:, None, :]
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


# ----------------------------------------------------------------------------- embedding

def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """The second table's row for every token: a hash of the token before and the token; the last row at the start."""
    return [buckets if t == 0 else (tokens[t - 1] * mul_prev + tokens[t] * mul_cur) % buckets for t in range(len(tokens))]


def embedding(w, cfg, tokens):
    e = cfg.get("embedding") or {}
    x = w["embed"][torch.tensor(tokens)] * e.get("scale", 1.0)
    b = e.get("bigram")
    if b:
        x = x + w["bigram"][torch.tensor(bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"]))]
    return x


# ----------------------------------------------------------------------------- attention with a window and pooled blocks

def seen_tokens(T, window):
    """[query, key]: keys up to the query itself, at most ``window`` of them (0: all)."""
    d = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (d >= 0) & ((d < window) if window else torch.ones_like(d, dtype=torch.bool))


def seen_blocks(T, window, pool):
    """[query, block]: blocks of ``pool`` tokens that lie wholly before the query's window."""
    last = torch.arange(T // pool) * pool + pool - 1
    return last[None, :] <= torch.arange(T)[:, None] - window


def block_means(x, pool):
    """x [T, ...]: the mean of every whole block of ``pool`` tokens."""
    n = x.shape[0] // pool
    return x[:n * pool].reshape((n, pool) + tuple(x.shape[1:])).mean(1)


def capped(score, cap):
    return cap * torch.tanh(score / cap) if cap else score


def pooled_sigmoid_attention(h, w, p, m, eps):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m.get("vdim", m["dim"])
    q = causal_conv(h @ w[p + ".q"].T, w[p + ".q.conv"])
    k = causal_conv(h @ w[p + ".k"].T, w[p + ".k.conv"])
    v = causal_conv(h @ w[p + ".v"].T, w[p + ".v.conv"])
    q = rms_norm(q, w[p + ".q.norm"], eps).view(T, H, d)             # over all heads at once
    k = rms_norm(k, w[p + ".k.norm"], eps).view(T, G, d)
    v = v.view(T, G, dv)
    mask = m.get("mask") or {}
    window, pool = mask.get("size", 0), mask.get("pool", 0)
    keys, values, seen = k, v, seen_tokens(T, window)
    if window and pool:
        keys = torch.cat((keys, block_means(k, pool)))
        values = torch.cat((values, block_means(v, pool)))
        seen = torch.cat((seen, seen_blocks(T, window, pool)), dim=1)
    out = torch.zeros(T, H, dv, dtype=F)
    for head in range(H):
        g = head // (H // G)
        score = capped((q[:, head] @ keys[:, g].T) * m["scale"], m.get("softcap", 0.0))
        weight = torch.sigmoid(score + w[p + ".pb"][head]) * seen    # nothing is normalised over the keys
        out[:, head] = weight @ values[:, g]
    return out.reshape(T, H * dv) @ w[p + ".o"].T


# ----------------------------------------------------------------------------- selective scan

def selective_scan(x, dt, A, B, C, D):
    """A row of states per channel: it decays by exp(dt A), takes in dt x B, is read out with C, and D passes x by."""
    T, inner = x.shape
    S = torch.zeros_like(A)
    y = torch.zeros_like(x)
    for t in range(T):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y


def mamba_mixer(h, w, p, m, eps=None):
    inner, N, R = m["inner"], m["state"], m["dt_rank"]
    u = h @ w[p + ".in"].T
    x, z = u[:, :inner], u[:, inner:]
    x = silu(causal_conv(x, w[p + ".conv"]) + w[p + ".conv.b"])
    proj = x @ w[p + ".x"].T
    dt, B, C = proj[:, :R], proj[:, R:R + N], proj[:, R + N:]
    dt = torch.nn.functional.softplus(dt @ w[p + ".dt"].T + w[p + ".dt.b"], threshold=1e9)
    y = selective_scan(x, dt, -torch.exp(w[p + ".A_log"]), B, C, w[p + ".D"])
    return (y * silu(z)) @ w[p + ".o"].T


def parallel_mixer(h, w, p, m, eps, shared):
    left = pooled_sigmoid_attention(h, w, p + ".left", m["left"], eps)
    right = mamba_mixer(h, w, p + ".right", m["right"])
    return m["left_scale"] * left + m["right_scale"] * right


# ----------------------------------------------------------------------------- latent attention

def latent_keys(h, w, p, m, eps):
    """(latent [T, kv_rank], rotated key part [T, rot_dim]): what a layer with ``dkv`` of its own keeps."""
    T, R, r = h.shape[0], m["kv_rank"], m["rot_dim"]
    down = h @ w[p + ".dkv"].T
    c = rms_norm(down[:, :R], w[p + ".dkv.norm"], eps)
    kr = down[:, R:]
    if r:
        kr = rotate_adjacent(kr.view(T, 1, r), torch.arange(T), r, m["rot"]["base"]).view(T, r)
    return c, kr


def latent_attention(h, w, p, m, eps, shared):
    T = h.shape[0]
    H, d, r, dv, R = m["heads"], m["dim"], m["rot_dim"], m.get("vdim", m["dim"]), m["kv_rank"]
    if m.get("kv_from") is None:
        shared[p] = latent_keys(h, w, p, m, eps)
        c, kr = shared[p]
    else:
        c, kr = shared[f"l{m['kv_from']}.mix"]
    q = (h @ w[p + ".q"].T).view(T, H, d + r)
    qp, qr = q[..., :d], q[..., d:]
    if r:
        qr = rotate_adjacent(qr, torch.arange(T), r, m["rot"]["base"])
    k = (c @ w[p + ".uk"].T).view(T, H, d)
    v = (c @ w[p + ".uv"].T).view(T, H, dv)
    seen = seen_tokens(T, (m.get("mask") or {}).get("size", 0))
    out = torch.zeros(T, H, dv, dtype=F)
    for head in range(H):
        score = (qp[:, head] @ k[:, head].T + qr[:, head] @ kr.T) * m["scale"]
        out[:, head] = torch.softmax(score.masked_fill(~seen, -math.inf), dim=-1) @ v[:, head]
    return (out.reshape(T, H * dv) * torch.sigmoid(h @ w[p + ".g"].T)) @ w[p + ".o"].T


MIXERS = {"parallel": parallel_mixer, "latent_attention": latent_attention}


# ----------------------------------------------------------------------------- routed feed-forward

MARGINS = None      # a list: every routed layer run appends, per token, how close its choice of groups or experts was


def choose_experts(s, top, groups, keep):
    """(indices of the ``top`` largest of the scores ``s`` [n] among the ``keep`` best of ``groups`` equal groups of
    neighbours, the smaller of the two gaps between what was taken and what was left: differences of the scores'
    logarithms, that is of the router's logits)."""
    gap = lambda a, b: math.log(a.item() / b.item()) if b.item() > 0 else math.inf        # noqa: E731
    n = s.numel()
    size = n // groups
    best = s.view(groups, size).max(-1).values
    order = sorted(range(groups), key=lambda g: (-best[g].item(), g))
    allowed = sorted(order[:keep])
    margin = math.inf if keep >= groups else gap(best[order[keep - 1]], best[order[keep]])
    cand = [e for g in allowed for e in range(g * size, (g + 1) * size)]
    cand.sort(key=lambda e: (-s[e].item(), e))
    if top < len(cand):
        margin = min(margin, gap(s[cand[top - 1]], s[cand[top]]))
    return cand[:top], margin


def clamped_unit(h, gate, up, down, limit):
    g = torch.clamp(h @ gate.T, max=limit)
    u = torch.clamp(h @ up.T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ down.T


def routed_ff(h, w, p, f):
    """Softmax scores over all experts, the choice limited to the best groups, weights = the chosen scores as they are."""
    r, limit = f["router"], f["expert"]["limit"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    s = torch.softmax(h @ w[p + ".router"].T, dim=-1)
    out, margins = torch.zeros_like(h), []
    for t in range(h.shape[0]):
        picked, margin = choose_experts(s[t], r["top"], groups["count"], groups["keep"])
        margins.append(margin)
        for e in picked:
            out[t] += s[t, e] * clamped_unit(h[t], w[f"{p}.e{e}.gate"], w[f"{p}.e{e}.up"], w[f"{p}.e{e}.down"], limit)
    if MARGINS is not None:
        MARGINS.append(torch.tensor(margins, dtype=F))
    return out


# ----------------------------------------------------------------------------- the model

def forward(w, cfg, tokens, layers_out=None, round_to=None):
    """Logits [T, vocab] of one sequence from its first token; ``layers_out`` receives the stream after every layer.
    With ``round_to`` every sublayer's input is rounded to that dtype on its way (what a model loses at the least when
    its products read such inputs)."""
    rounded = (lambda t: t.to(round_to).to(F)) if round_to is not None else (lambda t: t)
    eps = cfg["norm"]["eps"]
    x = embedding(w, cfg, list(tokens))
    shared = {}
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}"
        h = x + causal_conv(x, w[p + ".canon1"])
        y = MIXERS[L["type"]](rounded(h), w, p + ".mix", L["mixer"], eps, shared)
        x = x + rms_norm(y, 1 + w[p + ".norm1"], eps)
        if L.get("mlp"):
            x = x + rms_norm(routed_ff(rounded(x), w, p + ".mlp", L["mlp"]), 1 + w[p + ".norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return rounded(rms_norm(x, 1 + w["final.norm"], eps)) @ w["embed"].T


# ----------------------------------------------------------------------------- random weights

def tensor_shapes(cfg):
    """{tensor name: shape} of a model of this configuration."""
    W, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"]), "final.norm": (cfg["width"],)}
    b = (cfg.get("embedding") or {}).get("bigram")
    if b:
        out["bigram"] = (b["buckets"] + 1, W)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}", L["mixer"]
        out[p + ".norm1"] = (W,)
        out[p + ".canon1"] = (W, cfg["canon"]["taps"])
        q = p + ".mix"
        if L["type"] == "parallel":
            a, r = m["left"], m["right"]
            H, G, d, dv, taps = a["heads"], a["kv_heads"], a["dim"], a.get("vdim", a["dim"]), a["conv"]
            for s, n in (("q", H * d), ("k", G * d), ("v", G * dv)):
                out[f"{q}.left.{s}"], out[f"{q}.left.{s}.conv"] = (n, W), (n, taps)
            out.update({q + ".left.q.norm": (H * d,), q + ".left.k.norm": (G * d,), q + ".left.pb": (H,), q + ".left.o": (W, H * dv)})
            I, N, R = r["inner"], r["state"], r["dt_rank"]
            out.update({q + ".right.in": (2 * I, W), q + ".right.conv": (I, r["conv"]), q + ".right.conv.b": (I,),
                        q + ".right.x": (R + 2 * N, I), q + ".right.dt": (I, R), q + ".right.dt.b": (I,),
                        q + ".right.A_log": (I, N), q + ".right.D": (I,), q + ".right.o": (W, I)})
        else:
            H, d, r, dv, R = m["heads"], m["dim"], m["rot_dim"], m.get("vdim", m["dim"]), m["kv_rank"]
            out[q + ".q"] = (H * (d + r), W)
            if m.get("kv_from") is None:
                out.update({q + ".dkv": (R + r, W), q + ".dkv.norm": (R,)})
            out.update({q + ".uk": (H * d, R), q + ".uv": (H * dv, R), q + ".g": (H * dv, W), q + ".o": (W, H * dv)})
        f = L.get("mlp")
        if f:
            n, ff = f["router"]["experts"], f["expert"]["ff"]
            out.update({p + ".norm2": (W,), p + ".mlp.router": (n, W)})
            for e in range(n):
                out.update({f"{p}.mlp.e{e}.gate": (ff, W), f"{p}.mlp.e{e}.up": (ff, W), f"{p}.mlp.e{e}.down": (W, ff)})
    return out


def random_weights(cfg, seed, std=None):
    """bfloat16 tensors of a model of this configuration, sized so that every mechanism matters in the logits."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        r = torch.randn(shape, generator=g)
        if last in ("norm1", "norm2") or name == "final.norm":
            t = 0.2 * r                                              # a gain of one plus this
        elif last == "norm":
            t = 1.0 + 0.2 * r
        elif last == "canon1":
            t = 0.3 * r
        elif last == "conv":
            t = r / math.sqrt(shape[-1])
        elif last == "pb":
            t = -2.0 + r
        elif name.endswith("dt.b"):
            t = -3.0 + 1.5 * r
        elif last == "b":
            t = 0.3 * r
        elif last == "A_log":
            t = torch.log(torch.rand(shape, generator=g) * 8 + 0.1)
        elif last == "D":
            t = 1.0 + 0.3 * r
        elif last == "embed":
            t = 0.25 * r
        elif last == "bigram":
            t = 0.5 * r
        elif last == "router":
            t = r * 1.2 / math.sqrt(shape[-1])
        else:
            t = r * (std if std is not None else 1.2 / math.sqrt(shape[-1]))
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
