"""Plain, slow Funepel forward pass for tests: one function per mechanism.

Works on whole sequences (no cache, no batching, no fused weights, recurrences
token by token) with ordinary torch CPU operations in ``dtype`` (float64 by
default), straight from the config dictionary and the checkpoint tensors.
Shares no code with the package.  ``rnd`` rounds what a bf16 implementation may
round (operands and results of the projections and convolutions), so tests can
ask how much error rounding alone makes.
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


def dynamic_tanh(x, W, name):
    return torch.tanh(W[name + ".alpha"] * x) * W[name] + W[name + ".b"]


def silu(z):
    return z / (1 + torch.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(z.clamp(max=30))))


def positions(T, width, dtype):
    """(T, width): sin in the even entries, cos in the odd ones."""
    p = torch.arange(T, dtype=torch.float64)[:, None]
    out = torch.zeros(T, width, dtype=torch.float64)
    for c in range(width):
        a = p[:, 0] * 10000.0 ** (-2.0 * (c // 2) / width)
        out[:, c] = torch.sin(a) if c % 2 == 0 else torch.cos(a)
    return out.to(dtype)


def embed(tokens, table):
    return table[tokens] + positions(len(tokens), table.shape[1], table.dtype)


# ------------------------------------------------------------------ Mamba-2
def causal_conv(u, w, b):
    """u (T, C), w (C, taps) with the current token's tap last, zeros before the start."""
    T, taps = u.shape[0], w.shape[1]
    up = torch.cat([u.new_zeros(taps - 1, u.shape[1]), u])
    return sum(up[k:k + T] * w[:, k] for k in range(taps)) + b


def ssd(x, B, C, dt, a_log, d):
    """One head: x (T, P), B / C (T, N), dt (T,); S <- exp(-exp(a_log) dt) S + dt B x^T."""
    S = x.new_zeros(B.shape[1], x.shape[1])
    out = []
    for t in range(x.shape[0]):
        S = torch.exp(-torch.exp(a_log) * dt[t]) * S + dt[t] * torch.outer(B[t], x[t])
        out.append(S.t() @ C[t] + d * x[t])
    return torch.stack(out)


def gated_group_norm(y, z, w, groups, eps):
    """Gate first, then every one of ``groups`` equal parts by its own root mean square."""
    y = y * silu(z)
    return rms_norm(y.view(y.shape[0], groups, -1), eps).reshape(y.shape) * w


def mamba2_mixer(h, W, pre, m, eps, rnd=exact):
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    u = rnd(rnd(h) @ W[pre + "in"].t())
    z, xbc, dt = u[:, :inner], u[:, inner:2 * inner + 2 * G * N], u[:, 2 * inner + 2 * G * N:]
    xbc = rnd(silu(causal_conv(xbc, W[pre + "conv"], W[pre + "conv.b"])))
    dt = softplus(dt + W[pre + "dt_bias"])
    ys = []
    for n in range(H):
        g = n // (H // G)
        B = xbc[:, inner + g * N:inner + (g + 1) * N]
        C = xbc[:, inner + G * N + g * N:inner + G * N + (g + 1) * N]
        ys.append(ssd(xbc[:, n * P:(n + 1) * P], B, C, dt[:, n], W[pre + "A_log"][n], W[pre + "D"][n]))
    y = gated_group_norm(torch.cat(ys, -1), z, W[pre + "norm"], m["norm_groups"], eps)
    return rnd(rnd(y) @ W[pre + "o"].t())


# ------------------------------------------------------------------ attention beside retention
def visible(T, size):
    """(T, T) bool: query i (row) sees key j (column)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & (i - j < size)


def query_temperature(T, t):
    p = torch.arange(T, dtype=torch.float64)
    return 1 + t["coef"] * torch.log(torch.floor((p + 1) / t["every"]) + 1)


def slopes(H):
    return [2.0 ** (-8.0 * (h + 1) / H) for h in range(H)]


def biased_scores(q, k, scale, slope):
    """q, k (T, dim) of one query head: scaled dot products less slope * distance."""
    T = q.shape[0]
    dist = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(q.dtype)
    return (q @ k.t()) * scale - slope * dist


def masked_softmax(s, ok):
    s = s.masked_fill(~ok, -math.inf)
    p = torch.exp(s - s.max(-1, keepdim=True).values)
    return p / p.sum(-1, keepdim=True)


def attention_mixer(h, W, pre, m, eps, rnd=exact):
    H, G, dk = m["heads"], m["kv_heads"], m["dim"]
    T = h.shape[0]
    h = rnd(h)
    q, k = rnd(h @ W[pre + "q"].t()), rnd(h @ W[pre + "k"].t())
    v = k
    q, k = rms_norm(q, eps) * W[pre + "q.norm"], rms_norm(k, eps) * W[pre + "k.norm"]
    q = q * query_temperature(T, m["q_temp"]).to(q.dtype)[:, None]
    q, k = rnd(q), rnd(k)
    ok, sl = visible(T, m["mask"]["size"]), slopes(H)
    outs = []
    for n in range(H):
        c = n // (H // G)
        s = biased_scores(q[:, n * dk:(n + 1) * dk], k[:, c * dk:(c + 1) * dk], m["scale"], sl[n])
        outs.append(masked_softmax(s, ok) @ v[:, c * dk:(c + 1) * dk])
    o = torch.cat(outs, -1) * torch.sigmoid(rnd(h @ W[pre + "g"].t()))
    return rnd(rnd(o) @ W[pre + "o"].t())


def retention(q, k, v, decay):
    """One head: S <- decay S + k v^T, o = S^T q."""
    S = q.new_zeros(k.shape[1], v.shape[1])
    out = []
    for t in range(q.shape[0]):
        S = decay * S + torch.outer(k[t], v[t])
        out.append(S.t() @ q[t])
    return torch.stack(out)


def retention_mixer(h, W, pre, m, eps, rnd=exact):
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    h = rnd(h)
    q, k, v = (rnd(h @ W[pre + n].t()) for n in ("q", "k", "v"))
    k = k * dk ** -0.5
    o = [rms_norm(retention(q[:, n * dk:(n + 1) * dk], k[:, n * dk:(n + 1) * dk], v[:, n * dv:(n + 1) * dv],
                            m["decay"][n]), eps) for n in range(H)]
    y = torch.cat(o, -1) * silu(rnd(h @ W[pre + "g"].t()))
    return rnd(rnd(y) @ W[pre + "o"].t())


def parallel_mixer(h, W, pre, m, eps, rnd=exact):
    a = attention_mixer(h, W, pre + "left.", m["left"], eps, rnd)
    b = retention_mixer(h, W, pre + "right.", m["right"], eps, rnd)
    return 0.5 * (rms_norm(a, eps) * W[pre + "left.out"] + rms_norm(b, eps) * W[pre + "right.out"])


# ------------------------------------------------------------------ feed-forward
def gated_mlp(h, W, pre, rnd=exact):
    h = rnd(h)
    return rnd(rnd(silu(h @ W[pre + "gate"].t()) * (h @ W[pre + "up"].t())) @ W[pre + "down"].t())


def route(z, r):
    """z (T, experts) -> chosen experts (T, top) and their weights."""
    s = torch.softmax(z, -1)
    T, E = s.shape
    gr = r.get("groups")
    ok = torch.ones(T, E, dtype=torch.bool)
    if gr:
        best = s.view(T, gr["count"], -1).max(-1).values.topk(gr["keep"], -1).indices
        ok = torch.zeros(T, gr["count"], dtype=torch.bool).scatter(1, best, True)
        ok = ok.repeat_interleave(E // gr["count"], 1)
    w, idx = s.masked_fill(~ok, -1.0).topk(r["top"], -1)
    return idx, w / (w.sum(-1, keepdim=True) + 1e-20)


def moe(h, W, pre, m, rnd=exact):
    h = rnd(h)
    idx, w = route(h @ W[pre + "router"].t(), m["router"])
    y = torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        t, k = (idx == e).nonzero(as_tuple=True)
        if len(t):
            y[t] += w[t, k, None] * gated_mlp(h[t], W, f"{pre}e{e}.", rnd)
    if m.get("shared"):
        y = y + gated_mlp(h, W, pre + "shared.", rnd)
    return y


def side_input(x, e, W, pre, eps, rnd=exact):
    """Per-layer token input: e (T, side dim) this layer's part of the token's side embedding."""
    g = rnd(gelu_tanh(rnd(x) @ W[pre + "gate"].t()) * e)
    return rms_norm(rnd(g @ W[pre + "proj"].t()), eps) * W[pre + "norm"]


# ------------------------------------------------------------------ the model
def layer(x, tokens, i, cfg, W, rnd=exact):
    L, eps, p = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}."
    mixer = {"mamba2": mamba2_mixer, "parallel": parallel_mixer}[L["type"]]
    x = x + mixer(dynamic_tanh(x, W, p + "norm1"), W, p + "mix.", L["mixer"], eps, rnd)
    if L["mlp"] is not None:
        x = x + moe(dynamic_tanh(x, W, p + "norm2"), W, p + "mlp.", L["mlp"], rnd)
    if cfg.get("token_side"):
        d = cfg["token_side"]["dim"]
        e = W["side.embed"][tokens][:, i * d:(i + 1) * d]
        x = x + side_input(x, e, W, p + "side.", eps, rnd)
    return x


def layer_runs(cfg):
    """[(layer index, whether the embedding output is added first)] in the order of execution."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    runs = [(i, False) for i in range(lp["start"])]
    for t in range(lp["times"]):
        runs += [(i, t > 0 and i == lp["start"]) for i in range(lp["start"], lp["stop"])]
    return runs + [(i, False) for i in range(lp["stop"], n)]


def forward(tokens, cfg, W, trace=None, rnd=exact):
    """tokens (T,) -> logits (T, vocab); ``trace``: list that receives the residual after every layer run."""
    x = x0 = embed(tokens, W["embed"])
    for i, again in layer_runs(cfg):
        if again:
            x = x + x0
        x = layer(x, tokens, i, cfg, W, rnd)
        if trace is not None:
            trace.append(x)
    return rnd(rnd(dynamic_tanh(x, W, "final.norm")) @ W["head"].t())


# ------------------------------------------------------------------ weights
def tensor_shapes(cfg):
    """name -> shape of every tensor of a checkpoint with this config."""
    w = cfg["width"]
    s = {"embed": (cfg["vocab"], w), "head": (cfg["vocab"], w)}

    def norm(n):
        s[n], s[n + ".b"], s[n + ".alpha"] = (w,), (w,), ()

    def mlp(p, f):
        s[p + "gate"], s[p + "up"], s[p + "down"] = (f, w), (f, w), (w, f)
    norm("final.norm")
    sd = cfg["token_side"]["dim"] if cfg.get("token_side") else 0
    if sd:
        s["side.embed"] = (cfg["vocab"], sd * len(cfg["layers"]))
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        norm(p + "norm1")
        q = p + "mix."
        if L["type"] == "mamba2":
            H, inner = m["heads"], m["heads"] * m["vdim"]
            ch = inner + 2 * m["groups"] * m["state"]
            s.update({q + "in": (inner + ch + H, w), q + "conv": (ch, m["conv"]), q + "conv.b": (ch,),
                      q + "dt_bias": (H,), q + "A_log": (H,), q + "D": (H,), q + "norm": (inner,), q + "o": (w, inner)})
        else:
            a, b = m["left"], m["right"]
            nq, nk, r = a["heads"] * a["dim"], a["kv_heads"] * a["dim"], b["heads"]
            s.update({q + "left.q": (nq, w), q + "left.k": (nk, w), q + "left.q.norm": (nq,), q + "left.k.norm": (nk,),
                      q + "left.g": (nq, w), q + "left.o": (w, nq), q + "left.out": (w,)})
            s.update({q + "right.q": (r * b["dim"], w), q + "right.k": (r * b["dim"], w),
                      q + "right.v": (r * b["vdim"], w), q + "right.g": (r * b["vdim"], w),
                      q + "right.o": (w, r * b["vdim"]), q + "right.out": (w,)})
        if L["mlp"] is not None:
            norm(p + "norm2")
            for e in range(L["mlp"]["router"]["experts"]):
                mlp(f"{p}mlp.e{e}.", L["mlp"]["expert"]["ff"])
            s[p + "mlp.router"] = (L["mlp"]["router"]["experts"], w)
            if L["mlp"].get("shared"):
                mlp(p + "mlp.shared.", L["mlp"]["shared"]["ff"])
        if sd:
            s[p + "side.gate"], s[p + "side.proj"], s[p + "side.norm"] = (sd, w), (w, sd), (w,)
    return s


def random_weights(cfg, seed=0, gain=1.0):
    """bf16-representable float32 weights; scores, gates and norms of order one, so no mechanism is hidden."""
    g = torch.Generator().manual_seed(seed)
    W = {}
    for n, s in tensor_shapes(cfg).items():
        t = torch.randn(s, generator=g)
        if n.endswith(".alpha"):
            t = 0.6 + 0.1 * t
        elif n.endswith("dt_bias"):
            t = -1.5 + t
        elif n.endswith("A_log"):
            t = 0.7 * t
        elif n.endswith(".b"):
            t = 0.3 * t
        elif n.endswith("mix.conv"):
            t = t / math.sqrt(s[1])
        elif len(s) == 1:
            t = 1 + 0.2 * t
        elif n.endswith("mlp.router"):
            t = t * 2 / math.sqrt(s[1])
        elif len(s) == 2 and n not in ("embed", "side.embed"):
            t = t * gain / math.sqrt(s[1])
        W[n] = t.bfloat16().float()
    return W


def save_model(folder, cfg, W):
    from safetensors.torch import save_file
    with open(f"{folder}/config.json", "w") as f:
        json.dump(cfg, f)
    save_file({k: v.bfloat16().contiguous() for k, v in W.items()}, f"{folder}/model.safetensors")
