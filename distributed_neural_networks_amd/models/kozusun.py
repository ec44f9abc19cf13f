"""Kozusun: a decoder with parallel sublayers, a looped layer range, windowed
attention with kept first keys and a token input in every layer.

Per layer run, with the residual ``x`` in fp32, ``r`` = ``residual_mult`` and
``N(x; w) = x / sqrt(mean(x^2) + eps) * (1 + w)``:

    h  = N(x; norm1)
    x += r * (attention(h) + W_down (gelu_tanh(W_gate h) * W_up h))
    y  = W_proj (gelu_tanh(W_side x) * e_i[token])
    x += r * y / sqrt(mean(y^2) + eps) * side_norm

* attention: grouped-query, no rotation, biases on q / k / v, own score scale,
  value heads of their own size; query i sees key j when j <= i and
  (i - j < ``mask.size`` or j < ``mask.keep_first``); every head's output is
  multiplied by sigmoid of one projected number before the output projection.
* loop: layers ``start .. stop - 1`` run ``times`` times with shared weights and
  a cache of their own per pass; a pass begins with x <- W_in [x; x0], x0 the
  scaled embedding.
* e_i: part i of the token's row in a per-token table.

A model is a folder with ``config.json`` ("architecture": "Kozusun") and
safetensors weights (``embed``, ``loop.in``, ``side.embed``, ``l<i>.norm1``,
``l<i>.mix.{q,k,v,g,o}``, ``l<i>.mix.{q,k,v}.b``, ``l<i>.mlp.{gate,up,down}``,
``l<i>.side.{gate,proj,norm}``, ``final.norm``, ``head``), linear weights
``[out, in]``; every size and constant comes from the config.  Pipeline stages
split the sequence of layer *runs* (a looped layer counts once per pass).

This module holds the description only; ``runtime/decoder.py`` runs it.
"""
from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Dict, List, Optional, Tuple

from .decoder_config import (ModelConfigError, LayerRun, get_loop, get_number as _get, get_size as _size, layer_runs,
                             load_json)

ARCHITECTURE = "Kozusun"


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int] = None   # None: every earlier key
    keep_first: int = 0            # first keys that stay visible outside the window


@dataclass(frozen=True)
class LayerConfig:
    mixer: AttentionConfig
    ff: Optional[int]              # None: no feed-forward


@dataclass(frozen=True)
class KozusunConfig:
    vocab_size: int
    n_embd: int
    layers: Tuple[LayerConfig, ...]
    embed_scale: float
    norm_eps: float
    residual_mult: float
    loop: Optional[Tuple[int, int, int]] = None   # (start, stop, times)
    side_dim: int = 0                              # 0: no per-layer token input
    max_seq: int = 1 << 20                         # no positions enter the model: bounded by the cache only

    @property
    def n_layer(self) -> int:
        return len(self.runs)

    @property
    def runs(self) -> List[LayerRun]:
        return layer_runs(len(self.layers), self.loop, first_pass_enters=True)


def _attention(d, where) -> AttentionConfig:
    mask = d.get("mask")
    a = AttentionConfig(heads=_size(d, "heads", where), kv_heads=_size(d, "kv_heads", where),
                        dim=_size(d, "dim", where), vdim=_size(d, "vdim", where), scale=float(_get(d, "scale", where)),
                        window=_size(mask, "size", where + ".mask") if mask else None,
                        keep_first=int(mask.get("keep_first") or 0) if mask else 0)
    if a.heads % a.kv_heads:
        raise ModelConfigError(f"{where}: {a.heads} heads do not divide over {a.kv_heads} kv_heads")
    if not a.scale > 0 or a.keep_first < 0:
        raise ModelConfigError(f"{where}: 'scale' must be positive and 'keep_first' not negative")
    return a


def _layer(d, i) -> LayerConfig:
    where = f"layers[{i}]"
    if not isinstance(d, dict) or d.get("type") != "attention":
        raise ModelConfigError(f"{where}: unknown mixer type {d.get('type') if isinstance(d, dict) else d!r}")
    mlp = d.get("mlp")
    if mlp is not None and mlp.get("kind", "dense") != "dense":
        raise ModelConfigError(f"{where}: unknown feed-forward kind {mlp.get('kind')!r}")
    return LayerConfig(_attention(d.get("mixer") or {}, where + ".mixer"),
                       None if mlp is None else _size(mlp, "ff", where + ".mlp"))


def parse_config(d: Dict) -> KozusunConfig:
    if d.get("architecture") != ARCHITECTURE:
        raise ModelConfigError(f"architecture {d.get('architecture')!r} is not {ARCHITECTURE!r}")
    raw = d.get("layers")
    if not isinstance(raw, list) or not raw:
        raise ModelConfigError("'layers' must be a list with at least one layer")
    layers = tuple(_layer(x, i) for i, x in enumerate(raw))
    return KozusunConfig(vocab_size=_size(d, "vocab", "config"), n_embd=_size(d, "width", "config"), layers=layers,
                         embed_scale=float(_get(d.get("embedding"), "scale", "embedding")),
                         norm_eps=float(_get(d.get("norm"), "eps", "norm")),
                         residual_mult=float(_get(d, "residual_mult", "config")), loop=get_loop(d, len(layers)),
                         side_dim=_size(d["token_side"], "dim", "token_side") if d.get("token_side") else 0)


def load_config(folder: str) -> KozusunConfig:
    return load_json(folder, parse_config)


def make_config(vocab: int, width: int, n_layers: int, heads: int, kv_heads: int, dim: int, ff: Optional[int],
                window: Optional[int], keep_first: int = 0, vdim: Optional[int] = None, scale: Optional[float] = None,
                embed_scale: Optional[float] = None, residual_mult: float = 0.5, side_dim: int = 0,
                loop: Optional[Tuple[int, int, int]] = None, eps: float = 1e-5) -> KozusunConfig:
    """A config whose layers are all alike (presets, benches)."""
    att = AttentionConfig(heads, kv_heads, dim, vdim or dim, scale or dim ** -0.5, window, keep_first)
    return KozusunConfig(vocab, width, (LayerConfig(att, ff),) * n_layers, embed_scale or width ** 0.5, eps,
                         residual_mult, loop, side_dim)


KOZUSUN_CONFIGS: Dict[str, KozusunConfig] = {
    "kozusun-tiny": make_config(vocab=640, width=256, n_layers=4, heads=4, kv_heads=2, dim=64, ff=512, window=48,
                                keep_first=6, side_dim=32, loop=(1, 3, 2)),
    # layers of Llama-3 8B's size
    "kozusun-8b": make_config(vocab=128256, width=4096, n_layers=32, heads=32, kv_heads=8, dim=128, ff=14336,
                              window=4096, keep_first=64, side_dim=256),
    # layers of a 1B model's size, six of them looped
    "kozusun-1b": make_config(vocab=32768, width=2048, n_layers=16, heads=32, kv_heads=8, dim=64, ff=5632,
                              window=1024, keep_first=16, side_dim=128, loop=(4, 10, 2)),
}


def _layer_shapes(cfg: KozusunConfig, i: int) -> Dict[str, Tuple[int, ...]]:
    L, w, p = cfg.layers[i], cfg.n_embd, f"l{i}."
    m = L.mixer
    s: Dict[str, Tuple[int, ...]] = {p + "norm1": (w,)}
    for n, rows in (("q", m.heads * m.dim), ("k", m.kv_heads * m.dim), ("v", m.kv_heads * m.vdim)):
        s[p + f"mix.{n}"] = (rows, w)
        s[p + f"mix.{n}.b"] = (rows,)
    s[p + "mix.g"] = (m.heads, w)
    s[p + "mix.o"] = (w, m.heads * m.vdim)
    if L.ff is not None:
        s[p + "mlp.gate"], s[p + "mlp.up"], s[p + "mlp.down"] = (L.ff, w), (L.ff, w), (w, L.ff)
    if cfg.side_dim:
        s[p + "side.gate"], s[p + "side.proj"] = (cfg.side_dim, w), (w, cfg.side_dim)
        s[p + "side.norm"] = (w,)
    return s


def stage_shapes(cfg: KozusunConfig, start: int, end: int, first: bool, last: bool) -> Dict[str, Tuple[int, ...]]:
    """name -> shape of the tensors that layer runs ``start .. end`` need (checkpoint names)."""
    runs = cfg.runs[start:end + 1]
    s: Dict[str, Tuple[int, ...]] = {}
    enters = any(r.enters for r in runs)
    if first or enters:
        s["embed"] = (cfg.vocab_size, cfg.n_embd)
    if enters:
        s["loop.in"] = (cfg.n_embd, 2 * cfg.n_embd)
    if cfg.side_dim:
        s["side.embed"] = (cfg.vocab_size, cfg.side_dim * len(cfg.layers))
    for i in sorted({r.layer for r in runs}):
        s.update(_layer_shapes(cfg, i))
    if last:
        s["final.norm"], s["head"] = (cfg.n_embd,), (cfg.vocab_size, cfg.n_embd)
    return s


def stage_key_map(cfg: KozusunConfig, start: int, end: int, first: bool, last: bool) -> Dict[str, str]:
    return {k: k for k in stage_shapes(cfg, start, end, first, last)}


def random_tensor(cfg: KozusunConfig, name: str, noise, nontrivial: bool):
    """A random weight from unit ``noise`` of its shape: projections of unit
    gain, biases zero and norm weights one (stored around zero where the model
    adds the one), or noise around those with ``nontrivial``."""
    if noise.dim() == 1:
        extra = 0.1 * noise if nontrivial else 0 * noise
        return 1 + extra if name.endswith("side.norm") else extra
    if name == "embed":
        return noise / cfg.embed_scale
    return noise if name == "side.embed" else noise * noise.shape[1] ** -0.5


def run_flops(cfg: KozusunConfig, layer: int, ctx: int) -> float:
    """Forward FLOPs of one token through one run of ``layer`` with ``ctx`` keys before it."""
    L, m = cfg.layers[layer], cfg.layers[layer].mixer
    keys = ctx if m.window is None else min(ctx, m.window + m.keep_first)
    mats = sum(s[0] * s[1] for k, s in _layer_shapes(cfg, layer).items() if len(s) == 2)
    return 2.0 * mats + 2.0 * keys * m.heads * (m.dim + m.vdim)


def flops_per_token(cfg: KozusunConfig, runs: List[LayerRun], ctx: int, lm_head: bool = True) -> float:
    f = sum(run_flops(cfg, r.layer, ctx) + (4.0 * cfg.n_embd ** 2 if r.enters else 0.0) for r in runs)
    return f + (2.0 * cfg.n_embd * cfg.vocab_size if lm_head else 0.0)


def scaled(cfg: KozusunConfig, n_layers: int) -> KozusunConfig:
    """The same layers, ``n_layers`` of them, without a loop (benches)."""
    return replace(cfg, layers=cfg.layers[:1] * n_layers, loop=None)
