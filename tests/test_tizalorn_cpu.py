"""Tizalorn without a GPU: configuration, weights, packing of a step, and what
the oracle's inputs reveal."""
import copy
import math

import pytest
import torch

import tizalorn_oracle as O
from tizalorn_cases import CASES, config, latent, layer, moe, wkv

from distributed_neural_networks_amd import checkpoint as ckpt
from distributed_neural_networks_amd.config import parse_pipeline
from distributed_neural_networks_amd.models import build_golden_stage, default_ranges, model_info, tizalorn
from distributed_neural_networks_amd.ops import decoder_ops as D_
from distributed_neural_networks_amd.runtime.paging import KEY_ROWS, LatentHeads, PageTable, build_batch, tile_lists


# ------------------------------------------------------------------ configuration
@pytest.mark.parametrize("name", sorted(CASES))
def test_config_and_tensor_names(name):
    d = CASES[name]
    c = tizalorn.parse_config(d)
    n = c.n_layer
    assert [r.layer for r in c.runs] == list(range(n)) and not any(r.enters for r in c.runs)
    shapes, want = tizalorn.stage_shapes(c, 0, n - 1, True, True), O.tensor_shapes(d)
    assert set(shapes) == set(want) and all(ckpt.shape_fits(want[k], shapes[k]) for k in want)
    cut = max(1, n // 2)  # two stages together need every tensor, none of them twice
    parts = [tizalorn.stage_shapes(c, 0, cut - 1, True, False), tizalorn.stage_shapes(c, cut, n - 1, False, True)]
    assert set(parts[0]) | set(parts[1]) == set(want) and not set(parts[0]) & set(parts[1])
    assert all(tizalorn.run_flops(c, i, 100) > 0 for i in range(n))


@pytest.mark.parametrize("edit", [
    lambda d: d.update(architecture="Other"), lambda d: d.update(layers=[]), lambda d: d.pop("vocab"), lambda d: d.pop("norm"),
    lambda d: d.pop("embedding"), lambda d: d["embedding"]["bigram"].update(buckets=0),
    lambda d: d["embedding"]["bigram"].pop("mul_cur"),
    lambda d: d["layers"][0].update(type="other"), lambda d: d["layers"][0]["mlp"].update(kind="other"),
    lambda d: d["layers"][0]["mixer"].update(dim=257), lambda d: d["layers"][0]["mixer"].pop("heads"),
    lambda d: d["layers"][1]["mixer"].update(kv_rank=513), lambda d: d["layers"][1]["mixer"].update(rot_dim=18),
    lambda d: d["layers"][1]["mixer"]["rot"].update(dims=7), lambda d: d["layers"][1]["mixer"].pop("rot"),
    lambda d: d["layers"][1]["mixer"]["rot"].update(base=1.0), lambda d: d["layers"][1]["mixer"]["rot"]["scaling"].pop("fast"),
    lambda d: d["layers"][1]["mixer"]["rot"]["scaling"].update(factor=0), lambda d: d["layers"][1]["mixer"].update(scale=0),
    lambda d: d["layers"][1]["mlp"]["router"].update(top=7), lambda d: d["layers"][1]["mlp"]["router"]["groups"].update(count=4),
    lambda d: d["layers"][1]["mlp"]["router"]["groups"].update(keep=6), lambda d: d["layers"][1]["mlp"]["expert"].update(limit=0),
])
def test_config_errors(edit):
    d = copy.deepcopy(CASES["plain"])
    edit(d)
    with pytest.raises(tizalorn.ModelConfigError):
        tizalorn.parse_config(d)


def test_model_folder(tmp_path):
    d = CASES["mixed"]
    W = O.random_weights(d, 1)
    O.save_model(str(tmp_path), d, W)
    info = model_info(str(tmp_path))
    n = info.num_layers
    assert info.family == "tizalorn" and n == len(d["layers"])
    assert len(default_ranges(str(tmp_path), 2)) == 2
    sd = ckpt.stage_state_dict(info.name, ckpt.load_full_state_dict(str(tmp_path)), 0, n - 1, True, True)
    assert set(sd) == set(W) and all(torch.equal(sd[k].float(), W[k]) for k in W)
    assert sd["l0.norm1"].shape == () and "l2.norm2" not in sd
    with pytest.raises(ValueError, match="GPU"):
        build_golden_stage(info.name, 0, n - 1, True, True)
    bad = dict(sd)
    for k in ("l0.mlp.e3.down", "l1.mix.u", "l1.mix.w2"):
        bad[k] = bad[k][:-1]
        with pytest.raises(ckpt.CheckpointError, match=k.replace(".", r"\.")):
            ckpt.stage_state_dict(info.name, bad, 0, n - 1, True, True)
        bad[k] = sd[k]
    del bad["bigram"]
    with pytest.raises(ckpt.CheckpointError, match="missing"):
        ckpt.stage_state_dict(info.name, bad, 0, n - 1, True, True)
    pipe = {"nodes": [{"id": "n", "address": "127.0.0.1:5", "part_index": 0}], "model_weights": str(tmp_path),
            "num_parts": 1, "transport": "colocated", "model": str(tmp_path)}
    assert parse_pipeline(pipe).model == str(tmp_path)
    assert parse_pipeline(dict(pipe, model="tizalorn-tiny", model_weights="random")).model == "tizalorn-tiny"


def test_random_weights_are_stage_slices():
    n = model_info("tizalorn-tiny").num_layers
    full = ckpt.random_stage_state_dict("tizalorn-tiny", 0, n - 1, True, True, 3, nontrivial=True)
    part = ckpt.random_stage_state_dict("tizalorn-tiny", 2, n - 1, False, True, 3, nontrivial=True)
    assert part and all(torch.equal(full[k], v) for k, v in part.items())
    for name in ("tizalorn-1b", "tizalorn-8b"):
        c = model_info(name).cfg
        assert tizalorn.stage_shapes(c, 0, c.n_layer - 1, True, True)
    assert len(tizalorn.scaled(c, (1, 1, 3)).layers) == 3


# ------------------------------------------------------------------ packing
def test_step_rows_and_latent_tiles():
    """Every row knows its portion's first and last row; packed (token, head) rows
    of portions and of single tokens are dealt to workgroups apart."""
    t = PageTable(8, 4)
    s = [t.admit() for _ in range(4)]
    for x in s:
        t.reserve(x, 70)
    g = LatentHeads(40)
    b = build_batch([([7], 64, s[0], []), ([5, 6, 7], 3, s[1], []), ([1], 0, s[2], [0]), ([1, 2], 9, s[3], [])], t.table,
                    [g, 2], "cpu")
    assert b.start.tolist() == [0, 1, 1, 1, 4, 5, 5] and b.last.tolist() == [0, 3, 3, 3, 4, 6, 6]
    assert b.tiles[g, "chunks"].tolist() == [[1, 3, s[1], 64], [1, 3, s[1], 0], [5, 2, s[3], 64], [5, 2, s[3], 0]]
    assert b.tiles[g, "ones"].tolist() == [[0, 1, s[0], 0], [4, 1, s[2], 0]]
    assert [(LatentHeads(n).rows, LatentHeads(n).per_token) for n in (1, 32, 33, 64, 65)] == [(32, 1), (32, 1), (64, 1),
                                                                                           (64, 1), (64, 2)]
    assert all(v.data_ptr() % 16 == b.ids.data_ptr() % 16 for v in b.tiles.values())
    only = build_batch([([7], 64, s[0], [])], t.table, [g], "cpu")
    assert (g, "chunks") not in only.tiles


def test_portions_over_keys():
    """Long portions are scored over keys: their pages in rows of 64, as many as
    fit, the others over latents; unknown places stay over latents."""
    g = LatentHeads(2, 512, 128, 128, True)
    chunks, starts = [(0, 200, 3), (200, 31, 1), (231, 40, 0), (271, 40, 2)], [70, 0, 0, 5000]
    t = tile_lists([g], chunks, [(311, 1, 5)], starts)
    assert t[g, "keys"] == [(0, 200, 0, 128), (0, 200, 0, 0), (231, 40, 320, 0)]
    assert t[g, "pages"] == [(64 * i, 3, i, 0) for i in range(5)] + [(320, 0, 0, 0)]
    assert t[g, "chunks"] == [(200, 31, 1, 0), (271, 40, 2, 64), (271, 40, 2, 0)] and t[g, "ones"] == [(311, 1, 5, 0)]
    for other in (tile_lists([g], chunks, []), tile_lists([LatentHeads(2, 512, 128, 128)], chunks, [], starts)):
        assert [k for _, k in other] == ["chunks"]
    n = KEY_ROWS // 2
    two = tile_lists([g], [(0, n, 0), (n, n, 1), (2 * n, n, 2)], [], [0, 0, 0])  # the third does not fit
    assert len(two[g, "pages"]) == KEY_ROWS // 64 and {x[2] for x in two[g, "chunks"]} == {2}


def test_padding_rules():
    assert [D_.pad_to(n, D_.LATENT_DIMS, "x") for n in (1, 128, 129, 300, 512)] == [128, 128, 256, 512, 512]
    with pytest.raises(ValueError):
        D_.pad_to(513, D_.LATENT_DIMS, "x")
    assert D_.latent_splits(1, 1, 64) == 1 and D_.latent_splits(1, 1, 10000) > 8
    assert D_.latent_splits(300, 1, 10000) == 1 and D_.latent_ws(3, 2, 1, 128) == 0


# ------------------------------------------------------------------ what the inputs reveal
@pytest.mark.parametrize("scaling", [None, (4.0, 60, 6.0, 0.5), (1.0, 1, 1.0, 1.0), (8.0, 4096, 32.0, 1.0), (2.0, 3, 1.0, 1.0)])
def test_frequencies(scaling):
    m = latent(1, 1, 20, 1, 1, 1, 1.0, 700.0, scaling)[1]
    f, mag = tizalorn.parse_config(config([layer(("latent_attention", m))], 8, 8)).layers[0].mixer.rot.frequencies()
    rf, rmag = O.yarn_frequencies(m["rot"])
    assert f == pytest.approx(rf, rel=1e-14) and mag == pytest.approx(rmag, rel=1e-14)
    if scaling and scaling[1] == 60:  # fast pairs keep their frequency, slow ones are divided, some lie between
        r = [a * 700.0 ** (2 * i / 20) for i, a in enumerate(f)]
        assert r[0] == 1 and r[-1] == pytest.approx(0.25) and any(0.3 < x < 0.95 for x in r)
        assert mag == pytest.approx(1 + 0.1 * math.log(4))


def test_oracle_bigram_rows():
    b = {"buckets": 10, "mul_prev": 3, "mul_cur": 7}
    assert O.bigram_rows([4, 5, 9], b) == [10, (4 * 3 + 5 * 7) % 10, (5 * 3 + 9 * 7) % 10]


def test_oracle_router_groups():
    z, zero = torch.tensor([[3.0, 0.0, 2.0, 2.1, 2.9, -4.0]], dtype=torch.float64), torch.zeros(6, dtype=torch.float64)
    r = {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 1}}
    idx, w = O.route(z, zero, r)
    assert idx[0].tolist() == [3, 2]  # two good experts beat one of the best
    assert torch.allclose(w, torch.sigmoid(z[:, idx[0]]))  # as scored
    c = torch.tensor([0.0, 0, 0, 0, 0, 2], dtype=torch.float64)
    idx, w = O.route(z, c, r)
    assert idx[0].tolist() == [5, 4] and torch.allclose(w, torch.sigmoid(z[:, [5, 4]]))  # the correction chooses only
    idx, _ = O.route(z, zero - 3, r)
    assert idx[0].tolist() == [3, 2]  # negative choice scores are still better than a group that is out


def test_oracle_recurrence_is_the_quadratic_form():
    g = torch.Generator().manual_seed(0)
    r, k, v, la = (torch.randn(9, n, generator=g, dtype=torch.float64) for n in (4, 4, 3, 4))
    la, u = -la.abs(), torch.randn(4, generator=g, dtype=torch.float64)
    y = torch.zeros(9, 3, dtype=torch.float64)
    for t in range(9):
        for s in range(t):
            y[t] += (r[t] * k[s] * torch.exp(la[s + 1:t].sum(0))).sum() * v[s]
        y[t] += (r[t] * u * k[t]).sum() * v[t]
    assert torch.allclose(O.wkv(r, k, v, la, u), y)


def test_oracle_rotation_is_relative():
    """Scores of rotated parts depend on the distance only, up to the factor of cos and sin."""
    rot = latent(1, 1, 8, 1, 1, 1, 1.0)[1]["rot"]
    g = torch.Generator().manual_seed(1)
    q, k = (torch.randn(8, generator=g, dtype=torch.float64).expand(40, 8) for _ in range(2))
    s = O.rotate(q, rot) @ O.rotate(k, rot).t()
    assert torch.allclose(s.diagonal(), (q[0] @ k[0]) * O.yarn_frequencies(rot)[1] ** 2)
    assert torch.allclose(s[12, 5], s[39, 32]) and not torch.allclose(s[12, 5], s[5, 12])
    assert torch.equal(O.rotate(torch.ones(3, 10, dtype=torch.float64), rot)[:, 8:], torch.ones(3, 2, dtype=torch.float64))


def _att(d):
    return d["layers"][1]["mixer"]


def _roll_groups(z, c, r):
    """Groups scored by their best expert alone."""
    E, n = z.shape[1], z.shape[1] // r["groups"]["count"]
    s = O.sigmoid(z)
    best = (s + c).view(len(z), -1, n).amax(-1).topk(r["groups"]["keep"], -1).indices
    ok = torch.zeros(len(z), E // n, dtype=torch.bool).scatter(1, best, True).repeat_interleave(n, 1)
    idx = (s + c).masked_fill(~ok, -math.inf).topk(r["top"], -1).indices
    return idx, s.gather(1, idx)


def _both_sides(h, W, p, limit, rnd):
    """An expert whose gate is clamped from below as well."""
    g, u = (h @ W[p + "gate"].t()).clamp(-limit, limit), (h @ W[p + "up"].t()).clamp(-limit, limit)
    return (g * O.sigmoid(1.702 * g) * (u + 1)) @ W[p + "down"].t()


def _patched(name, make):
    """A mistake in the oracle's function ``name``."""
    return lambda d, W, mp: mp.setattr(O, name, make(getattr(O, name)))


def _edit(f):
    return lambda d, W, mp: f(d, W)


def _scaled(name, factor):
    return _edit(lambda d, W: W.update({name: W[name] * factor}))


MISTAKES = {
    "pair's tokens swapped": _edit(lambda d, W: d["embedding"]["bigram"].update(mul_prev=7, mul_cur=31)),
    "row of the first token": _patched("bigram_rows", lambda f: lambda t, b: [0] + f(t, b)[1:]),
    "token before of another portion": _patched("bigram_rows", lambda f: lambda t, b: f(t[:50], b) + f(t[50:], b)),
    "no embedding norm": _patched("embed", lambda f: lambda t, c, W: f(t, c, W) * 1.02),
    "portion starts without its token before": _patched(
        "token_shift", lambda f: lambda h, mu: torch.cat([f(h[:64], mu), f(h[64:], mu)])),
    "a mix of another stream": _edit(lambda d, W: W.update({"l0.mix.mu.r": W["l0.mix.mu.k"]})),
    "mix the wrong way round": _edit(lambda d, W: W.update({"l2.mix.mu.v": 1 - W["l2.mix.mu.v"]})),
    "decay without its bias": _scaled("l0.mix.w0", 0),
    "decay without its projection": _scaled("l2.mix.w2", 0),
    "decay of the next token": _patched("decay_log", lambda f: lambda *a: f(*a).roll(1, 0)),
    "state read after the update": _patched("wkv", lambda f: lambda r, k, v, la, u: f(r, k, v, la, u - u + 1)),
    "state lost at token 60": _patched("wkv", lambda f: lambda *a: torch.cat(
        [f(*(t[:60] for t in a[:4]), a[4]), f(*(t[60:] for t in a[:4]), a[4])])),
    "no bonus": _scaled("l0.mix.u", 0),
    "head norm's weight": _edit(lambda d, W: W.update({"l2.mix.norm": W["l2.mix.norm"].roll(64)})),
    "no recurrence gate": _scaled("l0.mix.g", 0.5),
    "rotation base": _edit(lambda d, W: _att(d)["rot"].update(base=750.0)),
    "frequencies not scaled": _edit(lambda d, W: _att(d)["rot"]["scaling"].update(factor=1.0)),
    "ramp a pair off": _edit(lambda d, W: _att(d)["rot"]["scaling"].update(original=90)),
    "no factor of cos and sin": _patched("yarn_frequencies", lambda f: lambda r: (f(r)[0], 1.0)),
    "halves instead of neighbours": _patched("rotate", lambda f: lambda x, r: torch.cat(
        [torch.stack([f(torch.stack([x[..., :10], x[..., 10:]], -1).flatten(-2), r)[..., i::2] for i in (0, 1)]).movedim(0, -2)
         .flatten(-2)], -1)),
    "positions one off": _patched("rotate", lambda f: lambda x, r: f(torch.cat([x[:1], x]), r)[1:] if x.dim() == 3 else f(x, r)),
    "score scale": _edit(lambda d, W: _att(d).update(scale=0.36)),
    "scale of the factor": _edit(lambda d, W: _att(d).update(scale=0.35 * (1 + 0.1 * math.log(4)) ** 2)),
    "query latent's norm weight": _edit(lambda d, W: W.update({"l1.mix.dq.norm": W["l1.mix.dq.norm"] * 0 + 1})),
    "latent's norm weight": _edit(lambda d, W: W.update({"l1.mix.dkv.norm": W["l1.mix.dkv.norm"] * 0 + 1})),
    "one key of the future": _patched("causal_softmax", lambda f: lambda s: torch.softmax(
        s.masked_fill(~torch.tril(torch.ones_like(s, dtype=torch.bool), 1), -math.inf), -1)),
    "first key left out": _patched("causal_softmax", lambda f: lambda s: torch.cat(
        [f(s)[:1], torch.nn.functional.pad(f(s[1:, 1:]), (1, 0))])),
    "no output gate": _scaled("l1.mix.g", 0),
    "gate of another head": _edit(lambda d, W: W.update({"l1.mix.g": W["l1.mix.g"].roll(1, 0)})),
    "powers of the norm": _patched("poly_norm", lambda f: lambda z, a, e: sum(
        a[i] * O.rms_norm(z, e) ** (i + 1) for i in range(3)) + a[3]),
    "no constant of the activation": _edit(lambda d, W: W.update({"l0.mlp.act": W["l0.mlp.act"] * torch.tensor([1., 1, 1, 0])})),
    "limit": _edit(lambda d, W: [x["mlp"].get("expert", {}).update(limit=1.0) for x in d["layers"]]),
    "gate clamped below too": _patched("expert", lambda f: _both_sides),
    "correction in the weights": _patched("route", lambda f: lambda z, c, r: (f(z, c, r)[0], f(z, c, r)[1] + c[f(z, c, r)[0]])),
    "no correction": _scaled("l1.mlp.correction", 0),
    "no groups of experts": _edit(lambda d, W: [x["mlp"].get("router", {}).pop("groups", None) for x in d["layers"]]),
    "groups by their best expert": _patched("route", lambda f: _roll_groups),
    "one expert less": _edit(lambda d, W: [x["mlp"].get("router", {}).update(top=2) for x in d["layers"]]),
    "norm weight": _scaled("l1.norm2", 1.05),
    "norms swapped": _edit(lambda d, W: W.update({"l0.norm1": W["l0.norm2"], "l0.norm2": W["l0.norm1"]})),
    "final norm": _scaled("final.norm", 1.01),
}


@pytest.mark.parametrize("name", sorted(MISTAKES))
def test_mistakes_show_in_logits(name, monkeypatch):
    """A mistake planted in the oracle moves the logits by far more than the
    tolerance of the GPU comparison: the random weights hide none."""
    d = copy.deepcopy(CASES["plain"])
    W = {k: v.double() for k, v in O.random_weights(d, 5, gain=1.5).items()}
    toks = torch.randint(0, d["vocab"], (90,), generator=torch.Generator().manual_seed(2)).tolist()
    ref = O.forward(toks, d, W)
    MISTAKES[name](d, W, monkeypatch)
    got = O.forward(toks, d, W)
    assert ((got - ref).norm() / ref.norm()).item() > 2e-3


def test_oracle_first_tokens_see_no_history():
    d = CASES["plain"]
    W = {k: v.double() for k, v in O.random_weights(d, 5).items()}
    toks = torch.randint(0, d["vocab"], (12,), generator=torch.Generator().manual_seed(1)).tolist()
    full = O.forward(toks, d, W)
    assert torch.allclose(full[:5], O.forward(toks[:5], d, W))
    assert not torch.allclose(full[5:6], O.forward(toks[5:6], d, W))


def test_case_helpers():
    c = tizalorn.parse_config(config([layer(wkv(2, 8), moe(2, 1, 8, 1.0))], 8, 8, (5, 12, -1)))
    assert c.layers[0].mixer.inner == 16 and c.layers[0].mlp.groups == 1 and c.layers[0].mlp.group_top == 2
    assert (c.bigram.mul_prev, c.bigram.mul_cur) == (2, 4)  # only the residues matter
