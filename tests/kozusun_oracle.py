"""Plain, slow Kozusun forward pass for tests: one function per mechanism.

Works on whole sequences (no cache, no batching, no fused weights) with
ordinary torch CPU operations in ``dtype`` (float64 by default), straight from
the config dictionary and the checkpoint tensors.  Shares no code with the
package.  ``rnd`` rounds what a bf16 implementation may round (operands and
results of the projections), so tests can ask how much error rounding alone
makes.
"""
from __future__ import annotations

import json
import math

import torch


def exact(t):
    return t


def bf16(t):
    return t.bfloat16().to(t.dtype)


def rms_norm(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last dim."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def zero_centred_norm(x, w, eps):
    return rms_norm(x, eps) * (1 + w)


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def embed(tokens, table, scale):
    return table[tokens] * scale


def visible(T, mask):
    """(T, T) bool: query i (row) sees key j (column)."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    ok = j <= i
    if mask is not None:
        ok = ok & (((i - j) < mask["size"]) | (j < mask.get("keep_first", 0)))
    return ok


def attention_scores(q, k, scale):
    """q (T, dim), k (T, dim) of one query head -> (T, T)."""
    return (q @ k.t()) * scale


def masked_softmax(s, ok):
    s = s.masked_fill(~ok, -math.inf)
    p = torch.exp(s - s.max(-1, keepdim=True).values)
    return p / p.sum(-1, keepdim=True)


def head_gate(h, wg):
    """(T, H): one factor per head and token."""
    return torch.sigmoid(h @ wg.t())


def attention_mixer(h, W, pre, m, rnd=exact):
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    h = rnd(h)
    q = rnd(h @ W[pre + "q"].t() + W[pre + "q.b"])
    k = rnd(h @ W[pre + "k"].t() + W[pre + "k.b"])
    v = rnd(h @ W[pre + "v"].t() + W[pre + "v.b"])
    g = head_gate(h, W[pre + "g"])
    ok = visible(T, m.get("mask"))
    outs = []
    for n in range(H):
        c = n // (H // G)
        s = attention_scores(q[:, n * dk:(n + 1) * dk], k[:, c * dk:(c + 1) * dk], m["scale"])
        outs.append(masked_softmax(s, ok) @ v[:, c * dv:(c + 1) * dv] * g[:, n:n + 1])
    return rnd(torch.cat(outs, -1)) @ W[pre + "o"].t()


def gated_mlp(h, W, pre, rnd=exact):
    h = rnd(h)
    return rnd(gelu_tanh(h @ W[pre + "gate"].t()) * (h @ W[pre + "up"].t())) @ W[pre + "down"].t()


def side_input(x, e, W, pre, eps, rnd=exact):
    """Per-layer token input: e (T, side dim) this layer's part of the token's side embedding."""
    g = rnd(gelu_tanh(rnd(rnd(x) @ W[pre + "gate"].t())) * e)
    return rms_norm(rnd(g @ W[pre + "proj"].t()), eps) * W[pre + "norm"]


def loop_in(x, x0, w, rnd=exact):
    return rnd(torch.cat([x, x0], -1)) @ w.t()


def layer(x, tokens, i, cfg, W, rnd=exact):
    L, eps, m = cfg["layers"][i], cfg["norm"]["eps"], cfg["residual_mult"]
    h = zero_centred_norm(x, W[f"l{i}.norm1"], eps)
    y = attention_mixer(h, W, f"l{i}.mix.", L["mixer"], rnd)
    if L["mlp"] is not None:
        y = y + gated_mlp(h, W, f"l{i}.mlp.", rnd)
    x = x + m * rnd(y)
    if cfg.get("token_side"):
        d = cfg["token_side"]["dim"]
        e = W["side.embed"][tokens][:, i * d:(i + 1) * d]
        x = x + m * side_input(x, e, W, f"l{i}.side.", eps, rnd)
    return x


def layer_runs(cfg):
    """[(layer index, whether a pass starts here)] in the order of execution."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    body = list(range(lp["start"], lp["stop"]))
    runs = [(i, False) for i in range(lp["start"])]
    for _ in range(lp["times"]):
        runs += [(i, i == body[0]) for i in body]
    return runs + [(i, False) for i in range(lp["stop"], n)]


def forward(tokens, cfg, W, trace=None, rnd=exact):
    """tokens (T,) -> logits (T, vocab); ``trace``: list that receives the residual after every layer run."""
    x = x0 = embed(tokens, W["embed"], cfg["embedding"]["scale"])
    for i, starts in layer_runs(cfg):
        if starts:
            x = loop_in(x, x0, W["loop.in"], rnd)
        x = layer(x, tokens, i, cfg, W, rnd)
        if trace is not None:
            trace.append(x)
    return rnd(rnd(zero_centred_norm(x, W["final.norm"], cfg["norm"]["eps"])) @ W["head"].t())


def tensor_shapes(cfg):
    """name -> shape of every tensor of a checkpoint with this config."""
    w, s = cfg["width"], {"embed": (cfg["vocab"], cfg["width"]), "final.norm": (cfg["width"],),
                          "head": (cfg["vocab"], cfg["width"])}
    if cfg.get("loop"):
        s["loop.in"] = (w, 2 * w)
    sd = cfg["token_side"]["dim"] if cfg.get("token_side") else 0
    if sd:
        s["side.embed"] = (cfg["vocab"], sd * len(cfg["layers"]))
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        s[p + "norm1"] = (w,)
        for n, r in (("q", H * dk), ("k", G * dk), ("v", G * dv)):
            s[p + f"mix.{n}"], s[p + f"mix.{n}.b"] = (r, w), (r,)
        s[p + "mix.g"], s[p + "mix.o"] = (H, w), (w, H * dv)
        if L["mlp"] is not None:
            f = L["mlp"]["ff"]
            s[p + "mlp.gate"], s[p + "mlp.up"], s[p + "mlp.down"] = (f, w), (f, w), (w, f)
        if sd:
            s[p + "side.gate"], s[p + "side.proj"], s[p + "side.norm"] = (sd, w), (w, sd), (w,)
    return s


def random_weights(cfg, seed=0, gain=1.0):
    """bf16-representable float32 weights; scores, gates and norms of order one, so no mechanism is hidden."""
    g = torch.Generator().manual_seed(seed)
    W = {}
    for n, s in tensor_shapes(cfg).items():
        t = torch.randn(s, generator=g)
        if n.endswith("norm1") or n == "final.norm":
            t = 0.2 * t
        elif n.endswith("side.norm"):
            t = 1 + 0.2 * t
        elif n.endswith(".b"):
            t = 0.3 * t
        elif n == "embed":
            t = t / cfg["embedding"]["scale"]
        elif len(s) == 2 and n != "side.embed":
            t = t * gain / math.sqrt(s[1])
        W[n] = t.bfloat16().float()
    return W


def save_model(folder, cfg, W):
    from safetensors.torch import save_file
    with open(f"{folder}/config.json", "w") as f:
        json.dump(cfg, f)
    save_file({k: v.bfloat16().contiguous() for k, v in W.items()}, f"{folder}/model.safetensors")
