"""What the paged decoder families (``kozusun.py``, ``funepel.py``,
``tizalorn.py``) share in their configurations: the folder's file name, checked reads of config.json, the
loop over a layer range, and the sequence of layer runs that pipeline stages
split.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Callable, Dict, List, Optional, Tuple

CONFIG_FILE = "config.json"


class ModelConfigError(ValueError):
    """config.json does not describe a model of this design."""


@dataclass(frozen=True)
class LayerRun:
    """One execution of a layer; ``enters``: the loop's entry step comes before it."""
    layer: int
    enters: bool


@dataclass(frozen=True)
class MoEConfig:
    """Mixture of experts: the router's scores (softmax, or sigmoid), a
    correction that enters the choice only, groups of neighbours scored by their
    ``group_top`` best experts, weights normalised over the chosen or as scored;
    ``limit``: experts with the clamped gated activation (g = min(gate, limit),
    u = clamp(up, +-limit), g sigmoid(alpha g) (u + shift)) instead of silu."""
    experts: int
    top: int
    ff: int
    groups: int = 1
    keep: int = 1
    shared_ff: int = 0      # 0: no shared expert
    sigmoid: bool = False
    correction: bool = False
    group_top: int = 1
    normalise: bool = True
    limit: Optional[float] = None
    alpha: float = 1.0
    shift: float = 0.0


def layer_runs(n: int, loop: Optional[Tuple[int, int, int]], first_pass_enters: bool) -> List[LayerRun]:
    """Runs of ``n`` layers whose range ``loop`` = (start, stop, times) repeats;
    ``first_pass_enters``: the first pass has an entry step too."""
    if loop is None:
        return [LayerRun(i, False) for i in range(n)]
    a, b, times = loop
    body = [LayerRun(i, i == a and (t > 0 or first_pass_enters)) for t in range(times) for i in range(a, b)]
    return [LayerRun(i, False) for i in range(a)] + body + [LayerRun(i, False) for i in range(b, n)]


def get_number(d, key, where, kinds=(int, float)):
    v = d.get(key) if isinstance(d, dict) else None
    if not isinstance(v, kinds) or isinstance(v, bool):
        raise ModelConfigError(f"{where}: '{key}' is missing or not a number, got {v!r}")
    return v


def get_size(d, key, where, low=1):
    v = get_number(d, key, where, (int,))
    if v < low:
        raise ModelConfigError(f"{where}: '{key}' must be >= {low}, got {v}")
    return v


def get_loop(d: Dict, n_layers: int) -> Optional[Tuple[int, int, int]]:
    if not d.get("loop"):
        return None
    a, b, t = (get_size(d["loop"], k, "loop", low) for k, low in (("start", 0), ("stop", 1), ("times", 1)))
    if not a < b <= n_layers:
        raise ModelConfigError(f"loop: layers {a} .. {b - 1} of {n_layers}")
    return a, b, t


def load_json(folder: str, parse: Callable):
    path = os.path.join(folder, CONFIG_FILE)
    try:
        with open(path) as f:
            return parse(json.load(f))
    except json.JSONDecodeError as e:
        raise ModelConfigError(f"{path}: {e}") from e
