"""Plain, slow Tizalorn forward pass for tests: one function per mechanism.

Works on whole sequences (no cache, no batching, no fused or absorbed weights,
the recurrence token by token) with ordinary torch CPU operations in ``dtype``
(float64 by default), straight from the config dictionary and the checkpoint
tensors.  Shares no code with the package.  ``rnd`` rounds what a bf16
implementation may round (operands and results of the projections), so tests
can ask how much error rounding alone makes.
"""
from __future__ import annotations

import json
import math

import torch


def exact(t):
    return t


def bf16(t):
    return t.bfloat16().to(t.dtype)


# ------------------------------------------------------------------ small functions
def rms_norm(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last dim."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def scalar_norm(x, W, name, eps):
    return rms_norm(x, eps) * W[name]


def silu(z):
    return z / (1 + torch.exp(-z))


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


# ------------------------------------------------------------------ embedding
def bigram_rows(tokens, b):
    """Row of the pair (previous token, token) in the bigram table; the last row for the first token."""
    rows = [b["buckets"]]
    for prev, cur in zip(tokens[:-1], tokens[1:]):
        rows.append((int(prev) * b["mul_prev"] + int(cur) * b["mul_cur"]) % b["buckets"])
    return rows


def embed(tokens, cfg, W):
    t = [int(i) for i in tokens]
    x = W["embed"][t] + W["bigram"][bigram_rows(t, cfg["embedding"]["bigram"])]
    return scalar_norm(x, W, "embed.norm", cfg["norm"]["eps"])


# ------------------------------------------------------------------ wkv
def token_shift(h, mu):
    """Every row mixed with the one before it (zeros before the first)."""
    prev = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (prev - h) * mu


def decay_log(m, W, pre, rnd=exact):
    """log of the decay of every head and key channel."""
    t = torch.tanh(rnd(m) @ W[pre + "w1"].t())
    return -torch.exp(t @ W[pre + "w2"].t() + W[pre + "w0"])


def wkv(r, k, v, la, u):
    """One head: r, k, la (T, D), v (T, D), u (D)."""
    S = r.new_zeros(k.shape[1], v.shape[1])
    out = []
    for t in range(r.shape[0]):
        kv = torch.outer(k[t], v[t])
        out.append((S + u[:, None] * kv).t() @ r[t])
        S = torch.exp(la[t])[:, None] * S + kv
    return torch.stack(out)


def wkv_mixer(h, W, pre, m, eps, rnd=exact):
    H, D = m["heads"], m["dim"]
    mix = {n: rnd(token_shift(h, W[pre + "mu." + n])) for n in "rkvgw"}
    r, k, v, g = (rnd(mix[n] @ W[pre + n].t()) for n in "rkvg")
    la = decay_log(mix["w"], W, pre, rnd)
    o = []
    for n in range(H):
        s = slice(n * D, (n + 1) * D)
        o.append(rms_norm(wkv(r[:, s], k[:, s], v[:, s], la[:, s], W[pre + "u"][n]), eps))
    y = torch.cat(o, -1) * W[pre + "norm"] * silu(g)
    return rnd(rnd(y) @ W[pre + "o"].t())


# ------------------------------------------------------------------ latent attention
def yarn_frequencies(rot):
    """Radians per position of every pair, and the factor of cos and sin."""
    d, base, f = rot["dims"], rot["base"], [rot["base"] ** (-2.0 * i / rot["dims"]) for i in range(rot["dims"] // 2)]
    s = rot.get("scaling")
    if not s:
        return f, 1.0

    def dim(turns):
        return d * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(dim(s["fast"])), 0), min(math.ceil(dim(s["slow"])), d - 1)
    out = []
    for i, x in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(x / s["factor"] * ramp + x * (1 - ramp))
    return out, 0.1 * math.log(s["factor"]) + 1


def rotate(x, rot):
    """x (T, ..., n): the first rot.dims values of the last dim as neighbouring pairs; row t is position t."""
    f, mag = yarn_frequencies(rot)
    out = x.clone()
    for t in range(x.shape[0]):
        for i, w in enumerate(f):
            c, s = math.cos(t * w) * mag, math.sin(t * w) * mag
            a, b = x[t, ..., 2 * i], x[t, ..., 2 * i + 1]
            out[t, ..., 2 * i], out[t, ..., 2 * i + 1] = a * c - b * s, b * c + a * s
    return out


def causal_softmax(s):
    T = s.shape[0]
    s = s.masked_fill(~torch.tril(torch.ones(T, T, dtype=torch.bool)), -math.inf)
    p = torch.exp(s - s.max(-1, keepdim=True).values)
    return p / p.sum(-1, keepdim=True)


def latent_attention_mixer(h, W, pre, m, eps, rnd=exact):
    H, D, R, V, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    T, h = h.shape[0], rnd(h)
    cq = rnd(rms_norm(rnd(h @ W[pre + "dq"].t()), eps) * W[pre + "dq.norm"])
    q = rnd(cq @ W[pre + "uq"].t()).view(T, H, D + R)
    kv = rnd(h @ W[pre + "dkv"].t())
    c, kr = rnd(rms_norm(kv[:, :C], eps) * W[pre + "dkv.norm"]), rnd(rotate(kv[:, C:], m["rot"]))
    qr = rnd(rotate(q[..., D:], m["rot"]))
    k, v = rnd(c @ W[pre + "uk"].t()).view(T, H, D), rnd(c @ W[pre + "uv"].t()).view(T, H, V)
    gate = sigmoid(rnd(h @ W[pre + "g"].t()))
    o = []
    for n in range(H):
        s = (q[:, n, :D] @ k[:, n].t() + qr[:, n] @ kr.t()) * m["scale"]
        o.append(causal_softmax(s) @ v[:, n] * gate[:, n:n + 1])
    return rnd(rnd(torch.cat(o, -1)) @ W[pre + "o"].t())


# ------------------------------------------------------------------ feed-forward
def poly_norm(z, act, eps):
    a, b, c, e = (act[i] for i in range(4))
    return a * rms_norm(z, eps) + b * rms_norm(z ** 2, eps) + c * rms_norm(z ** 3, eps) + e


def dense(h, W, pre, eps, rnd=exact):
    z = rnd(rnd(h) @ W[pre + "up"].t())
    return rnd(rnd(poly_norm(z, W[pre + "act"], eps)) @ W[pre + "down"].t())


def expert(h, W, pre, limit, rnd=exact):
    g = (h @ W[pre + "gate"].t()).clamp(max=limit)
    u = (h @ W[pre + "up"].t()).clamp(-limit, limit)
    return rnd(rnd(g * sigmoid(1.702 * g) * (u + 1)) @ W[pre + "down"].t())


def route(z, correction, r):
    """z (T, experts) -> chosen experts (T, top) and their weights."""
    s = sigmoid(z)
    choice = s + correction
    T, E = s.shape
    idx, gr = [], r.get("groups")
    for t in range(T):
        ok = list(range(E))
        if gr:
            n = E // gr["count"]
            score = [sum(sorted((float(choice[t, e]) for e in range(g * n, (g + 1) * n)), reverse=True)[:2])
                     for g in range(gr["count"])]
            best = sorted(range(gr["count"]), key=lambda g: (-score[g], g))[:gr["keep"]]
            ok = [e for e in ok if e // n in best]
        idx.append(sorted(ok, key=lambda e: (-float(choice[t, e]), e))[:r["top"]])
    idx = torch.tensor(idx)
    return idx, s.gather(1, idx)


def moe(h, W, pre, m, rnd=exact):
    h = rnd(h)
    idx, w = route(h @ W[pre + "router"].t(), W[pre + "correction"], m["router"])
    y = torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        t, k = (idx == e).nonzero(as_tuple=True)
        if len(t):
            y[t] += w[t, k, None] * expert(h[t], W, f"{pre}e{e}.", m["expert"]["limit"], rnd)
    return y


# ------------------------------------------------------------------ the model
def layer(x, i, cfg, W, rnd=exact):
    L, eps, p = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}."
    mixer = {"wkv": wkv_mixer, "latent_attention": latent_attention_mixer}[L["type"]]
    x = x + scalar_norm(mixer(x, W, p + "mix.", L["mixer"], eps, rnd), W, p + "norm1", eps)
    f = L.get("mlp")
    if f is not None:
        y = dense(x, W, p + "mlp.", eps, rnd) if f["kind"] == "dense" else moe(x, W, p + "mlp.", f, rnd)
        x = x + scalar_norm(y, W, p + "norm2", eps)
    return x


def forward(tokens, cfg, W, trace=None, rnd=exact):
    """tokens (T,) -> logits (T, vocab); ``trace``: list that receives the residual after every layer."""
    x = embed(tokens, cfg, W)
    for i in range(len(cfg["layers"])):
        x = layer(x, i, cfg, W, rnd)
        if trace is not None:
            trace.append(x)
    return rnd(rnd(scalar_norm(x, W, "final.norm", cfg["norm"]["eps"])) @ W["head"].t())


# ------------------------------------------------------------------ weights
def tensor_shapes(cfg, w1_rank=16):
    """name -> shape of every tensor of a checkpoint with this config (the decay's rank is a shape's only)."""
    w = cfg["width"]
    s = {"embed": (cfg["vocab"], w), "bigram": (cfg["embedding"]["bigram"]["buckets"] + 1, w), "embed.norm": (),
         "final.norm": (), "head": (cfg["vocab"], w)}
    for i, L in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L.get("mlp")
        s[p + "norm1"], q = (), p + "mix."
        if L["type"] == "wkv":
            n = m["heads"] * m["dim"]
            for x in "rkvgw":
                s[q + "mu." + x] = (w,)
            for x in "rkvg":
                s[q + x] = (n, w)
            s.update({q + "w1": (w1_rank, w), q + "w2": (n, w1_rank), q + "w0": (n,), q + "u": (m["heads"], m["dim"]),
                      q + "norm": (n,), q + "o": (w, n)})
        else:
            H, D, R, V, C, Q = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
            s.update({q + "dq": (Q, w), q + "dq.norm": (Q,), q + "uq": (H * (D + R), Q), q + "dkv": (C + R, w),
                      q + "dkv.norm": (C,), q + "uk": (H * D, C), q + "uv": (H * V, C), q + "g": (H, w),
                      q + "o": (w, H * V)})
        if f is None:
            continue
        s[p + "norm2"], q = (), p + "mlp."
        if f["kind"] == "dense":
            s.update({q + "up": (f["ff"], w), q + "down": (w, f["ff"]), q + "act": (4,)})
        else:
            E, F = f["router"]["experts"], f["expert"]["ff"]
            s[q + "router"], s[q + "correction"] = (E, w), (E,)
            for e in range(E):
                s.update({f"{q}e{e}.gate": (F, w), f"{q}e{e}.up": (F, w), f"{q}e{e}.down": (w, F)})
    return s


def random_weights(cfg, seed=0, gain=1.0, w1_rank=16):
    """bf16-representable float32 weights; scores, gates, decays and norms spread so that no mechanism is hidden."""
    g = torch.Generator().manual_seed(seed)
    W = {}
    for n, s in tensor_shapes(cfg, w1_rank).items():
        t = torch.randn(s, generator=g)
        if n.endswith(("norm1", "norm2", "embed.norm", "final.norm")):
            t = 0.9 + 0.2 * t.abs()
        elif n.endswith("mlp.act"):
            t = torch.tensor([0.7, 0.5, -0.4, 0.2]) + 0.1 * t
        elif n.endswith("mlp.correction"):
            t = 0.4 * t - 0.5          # choice scores of either sign
        elif ".mu." in n:
            t = 0.5 + 0.3 * t
        elif n.endswith("mix.w0"):
            t = 1.8 * t - 2.5          # memories of one to a few hundred tokens
        elif n.endswith("mix.w2"):
            t = t / math.sqrt(s[1])
        elif n.endswith("mix.u"):
            t = 0.5 + 0.5 * t.abs()
        elif len(s) == 1:
            t = 1 + 0.2 * t
        elif n.endswith("mlp.router"):
            t = t * 1.5 / math.sqrt(s[1])
        elif n not in ("embed", "bigram"):
            t = t * gain / math.sqrt(s[1])
        W[n] = t.bfloat16().float()
    # A head's output is normed, so a first token whose r . (u k) is near zero
    # would turn rounding into another sign: r and k point the same way.
    for i, L in enumerate(cfg["layers"]):
        if L["type"] == "wkv":
            p = f"l{i}.mix."
            for a, b in ((p + "mu.k", p + "mu.r"), (p + "k", p + "r")):
                W[a] = (0.6 * W[a] + 0.6 * W[b]).bfloat16().float()
    return W


def save_model(folder, cfg, W):
    from safetensors.torch import save_file
    with open(f"{folder}/config.json", "w") as f:
        json.dump(cfg, f)
    save_file({k: v.bfloat16().contiguous() for k, v in W.items()}, f"{folder}/model.safetensors")
