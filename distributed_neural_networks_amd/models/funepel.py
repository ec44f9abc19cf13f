"""Funepel: a decoder of recurrent layers and layers that run attention beside
retention, each followed by a mixture of experts and a token input, with a
looped layer range.

The residual ``x`` is fp32; ``DyT(x; w) = tanh(alpha x) * w + b``, ``N(y) = y /
sqrt(mean(y^2) + eps)``:

    x  = embed[token] + sinusoidal position vector              (also x0)
    x += mixer(DyT(x; norm1));  x += experts(DyT(x; norm2))
    x += N(W_proj (gelu_tanh(W_side x) * e_i[token])) * side_norm

* loop: layers ``start .. stop - 1`` run ``times`` times with shared weights, a
  cache or state of their own per pass; every pass but the first begins with
  x <- x + x0.
* mixer ``mamba2``: a projection to [z | x | B | C | dt], a short causal
  convolution with silu over x, B and C, the state-space recurrence
  S <- exp(-exp(A_log) dt) S + dt B x^T, y = S^T C + D x per head (groups of
  heads share B and C), then y * silu(z), RMS norm of equal parts, W_o.
* mixer ``parallel``: attention and retention read the same input; their
  outputs are RMS-normed over the width and averaged.  Attention: grouped
  queries, norm over whole q / k projections, a query temperature that grows
  with the logarithm of the position, keys that are the values too, a linear
  distance bias, a sliding window, an output gate per element.  Retention: a
  linear recurrence with one fixed decay per head, the heads RMS-normed, gated
  by silu.
* experts: softmax router, the best groups of neighbours, the best experts in
  them, weights normalised; a shared expert runs for every token.

A model is a folder with ``config.json`` ("architecture": "Funepel") and
safetensors weights named ``embed``, ``side.embed``, ``l<i>.norm{1,2}[.b,
.alpha]``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``l<i>.side.*``, ``final.norm[...]``,
``head``; linear weights ``[out, in]``; every size and constant comes from the
config.  Pipeline stages split the sequence of layer *runs*.

This module holds the description only; ``runtime/decoder.py`` runs it.
"""
from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Dict, List, Optional, Tuple, Union

from .decoder_config import (MoEConfig, ModelConfigError, LayerRun, get_loop, get_number as _get, get_size as _size, layer_runs,
                             load_json)

ARCHITECTURE = "Funepel"
STATE_MAX = 256    # state rows (key sizes) the recurrence kernels are built for
EXPERTS_MAX = 256


@dataclass(frozen=True)
class Mamba2Config:
    heads: int
    vdim: int
    state: int
    groups: int        # heads // groups heads share B and C
    conv: int          # taps
    norm_groups: int   # parts of the gated norm

    @property
    def inner(self) -> int:
        return self.heads * self.vdim


@dataclass(frozen=True)
class SharedKVAttentionConfig:
    """Attention whose values are its keys, with a norm over whole projections."""
    heads: int
    kv_heads: int
    dim: int
    scale: float
    window: Optional[int]   # None: every earlier key
    temp_coef: float = 0.0
    temp_every: int = 0     # 0: no query temperature
    keep_first: int = 0


@dataclass(frozen=True)
class RetentionConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]


@dataclass(frozen=True)
class ParallelConfig:
    left: SharedKVAttentionConfig
    right: RetentionConfig


@dataclass(frozen=True)
class LayerConfig:
    mixer: Union[Mamba2Config, ParallelConfig]
    mlp: Optional[MoEConfig]


@dataclass(frozen=True)
class FunepelConfig:
    vocab_size: int
    n_embd: int
    layers: Tuple[LayerConfig, ...]
    norm_eps: float
    loop: Optional[Tuple[int, int, int]] = None   # (start, stop, times)
    side_dim: int = 0                              # 0: no per-layer token input
    max_seq: int = 1 << 20                         # bounded by the cache only

    @property
    def n_layer(self) -> int:
        return len(self.runs)

    @property
    def runs(self) -> List[LayerRun]:
        return layer_runs(len(self.layers), self.loop, first_pass_enters=False)


def _divides(a: int, b: int, what: str, where: str) -> None:
    if a % b:
        raise ModelConfigError(f"{where}: {what}: {a} does not divide over {b}")


def _mamba2(d, where) -> Mamba2Config:
    m = Mamba2Config(**{k: _size(d, k, where) for k in ("heads", "vdim", "state", "groups", "conv", "norm_groups")})
    _divides(m.heads, m.groups, "heads over groups", where)
    _divides(m.inner, m.norm_groups, "heads * vdim over norm_groups", where)
    if m.state > STATE_MAX:
        raise ModelConfigError(f"{where}: 'state' {m.state} exceeds {STATE_MAX}")
    return m


def _attention(d, where) -> SharedKVAttentionConfig:
    t = d.get("q_temp")
    a = SharedKVAttentionConfig(heads=_size(d, "heads", where), kv_heads=_size(d, "kv_heads", where),
                                dim=_size(d, "dim", where), scale=float(_get(d, "scale", where)),
                                window=_size(d["mask"], "size", where + ".mask") if d.get("mask") else None,
                                temp_coef=float(_get(t, "coef", where + ".q_temp")) if t else 0.0,
                                temp_every=_size(t, "every", where + ".q_temp") if t else 0)
    _divides(a.heads, a.kv_heads, "heads over kv_heads", where)
    if d.get("vdim", a.dim) != a.dim:
        raise ModelConfigError(f"{where}: the values are the keys, but 'vdim' {d['vdim']} is not 'dim' {a.dim}")
    if not a.scale > 0:
        raise ModelConfigError(f"{where}: 'scale' must be positive")
    return a


def _retention(d, where) -> RetentionConfig:
    decay = d.get("decay")
    heads = _size(d, "heads", where)
    if not isinstance(decay, list) or len(decay) != heads or not all(
            isinstance(x, (int, float)) and not isinstance(x, bool) and 0 <= x <= 1 for x in decay):
        raise ModelConfigError(f"{where}: 'decay' must list a number in [0, 1] for each of the {heads} heads")
    r = RetentionConfig(heads, _size(d, "dim", where), _size(d, "vdim", where), tuple(float(x) for x in decay))
    if r.dim > STATE_MAX:
        raise ModelConfigError(f"{where}: 'dim' {r.dim} exceeds {STATE_MAX}")
    return r


def _moe(d, where) -> MoEConfig:
    if d.get("kind", "moe") != "moe":
        raise ModelConfigError(f"{where}: unknown feed-forward kind {d.get('kind')!r}")
    r, g, shared = d.get("router") or {}, (d.get("router") or {}).get("groups"), d.get("shared")
    m = MoEConfig(experts=_size(r, "experts", where + ".router"), top=_size(r, "top", where + ".router"),
                  ff=_size(d.get("expert"), "ff", where + ".expert"),
                  groups=_size(g, "count", where + ".router.groups") if g else 1,
                  keep=_size(g, "keep", where + ".router.groups") if g else 1,
                  shared_ff=_size(shared, "ff", where + ".shared") if shared else 0)
    _divides(m.experts, m.groups, "experts over groups", where)
    if m.keep > m.groups or m.top > m.experts // m.groups * m.keep or m.experts > EXPERTS_MAX or m.top > 64:
        raise ModelConfigError(f"{where}: {m.top} of {m.experts} experts from {m.keep} of {m.groups} groups")
    return m


def _layer(d, i) -> LayerConfig:
    where = f"layers[{i}]"
    kind, m = (d.get("type"), d.get("mixer") or {}) if isinstance(d, dict) else (d, {})
    if kind == "mamba2":
        mixer = _mamba2(m, where + ".mixer")
    elif kind == "parallel":
        mixer = ParallelConfig(_attention(m.get("left") or {}, where + ".mixer.left"),
                               _retention(m.get("right") or {}, where + ".mixer.right"))
    else:
        raise ModelConfigError(f"{where}: unknown mixer type {kind!r}")
    return LayerConfig(mixer, None if d.get("mlp") is None else _moe(d["mlp"], where + ".mlp"))


def parse_config(d: Dict) -> FunepelConfig:
    if d.get("architecture") != ARCHITECTURE:
        raise ModelConfigError(f"architecture {d.get('architecture')!r} is not {ARCHITECTURE!r}")
    raw = d.get("layers")
    if not isinstance(raw, list) or not raw:
        raise ModelConfigError("'layers' must be a list with at least one layer")
    layers = tuple(_layer(x, i) for i, x in enumerate(raw))
    return FunepelConfig(vocab_size=_size(d, "vocab", "config"), n_embd=_size(d, "width", "config"), layers=layers,
                         norm_eps=float(_get(d.get("norm"), "eps", "norm")), loop=get_loop(d, len(layers)),
                         side_dim=_size(d["token_side"], "dim", "token_side") if d.get("token_side") else 0)


def load_config(folder: str) -> FunepelConfig:
    return load_json(folder, parse_config)


def retention_decays(heads: int, low: float = 5.0) -> Tuple[float, ...]:
    """1 - 2^-(low .. low + 5): memories of tens to a thousand tokens."""
    return tuple(1.0 - 2.0 ** -(low + 5.0 * h / max(1, heads - 1)) for h in range(heads))


FUNEPEL_CONFIGS: Dict[str, FunepelConfig] = {}


def _preset(name: str, vocab: int, width: int, pattern: str, mamba: Mamba2Config, par: ParallelConfig, moe: MoEConfig,
            side_dim: int, loop=None) -> None:
    layers = tuple(LayerConfig(mamba if c == "m" else par, moe) for c in pattern)
    FUNEPEL_CONFIGS[name] = FunepelConfig(vocab, width, layers, 1e-6, loop, side_dim)


_preset("funepel-tiny", 640, 192, "mpm", Mamba2Config(6, 32, 64, 2, 4, 3),
        ParallelConfig(SharedKVAttentionConfig(6, 2, 64, 0.125, 80, 0.2, 32), RetentionConfig(3, 48, 64, retention_decays(3))),
        MoEConfig(12, 3, 96, 3, 2, 128), side_dim=32, loop=(0, 2, 2))
# layers of a 1B model's and of Llama-3 8B's width; active feed-forward columns near theirs
_preset("funepel-1b", 32768, 2048, "mpppmppp", Mamba2Config(64, 64, 128, 8, 4, 8),
        ParallelConfig(SharedKVAttentionConfig(32, 8, 64, 0.125, 1024, 0.1, 4096),
                       RetentionConfig(16, 128, 128, retention_decays(16))),
        MoEConfig(32, 4, 1024, 4, 2, 1536), side_dim=128, loop=(1, 4, 2))
_preset("funepel-8b", 128256, 4096, "mppp" * 4, Mamba2Config(128, 64, 128, 8, 4, 8),
        ParallelConfig(SharedKVAttentionConfig(32, 8, 128, 128 ** -0.5, 4096, 0.1, 8192),
                       RetentionConfig(16, 256, 256, retention_decays(16))),
        MoEConfig(32, 4, 2816, 4, 2, 3072), side_dim=256)


def _layer_shapes(cfg: FunepelConfig, i: int) -> Dict[str, Tuple[int, ...]]:
    L, w, p = cfg.layers[i], cfg.n_embd, f"l{i}."
    s: Dict[str, Tuple[int, ...]] = {}

    def norm(n):
        s[n], s[n + ".b"], s[n + ".alpha"] = (w,), (w,), ()

    def gated(n, ff):
        s[n + ".gate"], s[n + ".up"], s[n + ".down"] = (ff, w), (ff, w), (w, ff)
    norm(p + "norm1")
    m, q = L.mixer, p + "mix."
    if isinstance(m, Mamba2Config):
        ch = m.inner + 2 * m.groups * m.state
        s[q + "in"] = (m.inner + ch + m.heads, w)
        s[q + "conv"], s[q + "conv.b"] = (ch, m.conv), (ch,)
        s[q + "dt_bias"] = s[q + "A_log"] = s[q + "D"] = (m.heads,)
        s[q + "norm"], s[q + "o"] = (m.inner,), (w, m.inner)
    else:
        a, r = m.left, m.right
        nq, nk = a.heads * a.dim, a.kv_heads * a.dim
        s[q + "left.q"], s[q + "left.k"], s[q + "left.g"], s[q + "left.o"] = (nq, w), (nk, w), (nq, w), (w, nq)
        s[q + "left.q.norm"], s[q + "left.k.norm"], s[q + "left.out"] = (nq,), (nk,), (w,)
        rk, rv = r.heads * r.dim, r.heads * r.vdim
        s[q + "right.q"] = s[q + "right.k"] = (rk, w)
        s[q + "right.v"] = s[q + "right.g"] = (rv, w)
        s[q + "right.o"], s[q + "right.out"] = (w, rv), (w,)
    if L.mlp is not None:
        norm(p + "norm2")
        for e in range(L.mlp.experts):
            gated(f"{p}mlp.e{e}", L.mlp.ff)
        s[p + "mlp.router"] = (L.mlp.experts, w)
        if L.mlp.shared_ff:
            gated(p + "mlp.shared", L.mlp.shared_ff)
    if cfg.side_dim:
        s[p + "side.gate"], s[p + "side.proj"] = (cfg.side_dim, w), (w, cfg.side_dim)
        s[p + "side.norm"] = (w,)
    return s


def stage_shapes(cfg: FunepelConfig, start: int, end: int, first: bool, last: bool) -> Dict[str, Tuple[int, ...]]:
    """name -> shape of the tensors that layer runs ``start .. end`` need (checkpoint names)."""
    runs = cfg.runs[start:end + 1]
    s: Dict[str, Tuple[int, ...]] = {}
    if first or any(r.enters for r in runs):
        s["embed"] = (cfg.vocab_size, cfg.n_embd)
    if cfg.side_dim:
        s["side.embed"] = (cfg.vocab_size, cfg.side_dim * len(cfg.layers))
    for i in sorted({r.layer for r in runs}):
        s.update(_layer_shapes(cfg, i))
    if last:
        s["final.norm"] = s["final.norm.b"] = (cfg.n_embd,)
        s["final.norm.alpha"], s["head"] = (), (cfg.vocab_size, cfg.n_embd)
    return s


def stage_key_map(cfg: FunepelConfig, start: int, end: int, first: bool, last: bool) -> Dict[str, str]:
    return {k: k for k in stage_shapes(cfg, start, end, first, last)}


def random_tensor(cfg: FunepelConfig, name: str, noise, nontrivial: bool):
    """A random weight from unit ``noise`` of its shape: projections of unit
    gain, norm weights one (biases zero), or noise around those with
    ``nontrivial``; decays of a few to a few hundred tokens."""
    shape, extra = tuple(noise.shape), 0.1 * noise if nontrivial else 0 * noise
    if name.endswith(".alpha"):
        return 0.7 + extra
    if name.endswith("dt_bias"):
        return noise - 2.0
    if name.endswith("A_log"):
        return 0.5 * noise
    if name.endswith(".b"):
        return extra
    if len(shape) == 1:
        return 1 + extra
    if name in ("embed", "side.embed"):
        return noise
    return noise * shape[1] ** -0.5


def run_flops(cfg: FunepelConfig, layer: int, ctx: int) -> float:
    """Forward FLOPs of one token through one run of ``layer`` with ``ctx`` tokens before it."""
    L, m = cfg.layers[layer], cfg.layers[layer].mixer
    idle = f"l{layer}.mlp.e"
    mats = sum(s[0] * s[1] for k, s in _layer_shapes(cfg, layer).items()
               if len(s) == 2 and not k.startswith(idle) and not k.endswith("mix.conv"))
    if L.mlp is not None:
        mats += 3 * L.mlp.top * L.mlp.ff * cfg.n_embd
    if isinstance(m, Mamba2Config):
        mix = 4.0 * m.inner * m.state + 2.0 * m.conv * (m.inner + 2 * m.groups * m.state)
    else:
        keys = ctx if m.left.window is None else min(ctx, m.left.window)
        mix = 4.0 * keys * m.left.heads * m.left.dim + 4.0 * m.right.heads * m.right.dim * m.right.vdim
    return 2.0 * mats + mix


def flops_per_token(cfg: FunepelConfig, runs: List[LayerRun], ctx: int, lm_head: bool = True) -> float:
    f = sum(run_flops(cfg, r.layer, ctx) for r in runs)
    return f + (2.0 * cfg.n_embd * cfg.vocab_size if lm_head else 0.0)


def scaled(cfg: FunepelConfig, pattern: Tuple[int, ...]) -> FunepelConfig:
    """The layers ``pattern`` of ``cfg``, without a loop (benches)."""
    return replace(cfg, layers=tuple(cfg.layers[i] for i in pattern), loop=None)
