"""Kozusun without a GPU: configuration, weights, page bookkeeping, the engine's
scheduling (over a stand-in stage), and what the oracle's inputs reveal."""
import copy
import io
import json
import math

import numpy as np
import pytest
import torch

import kozusun_oracle as O
from kozusun_cases import CASES, att, config, layer

from distributed_neural_networks_amd import checkpoint as ckpt
from distributed_neural_networks_amd.config import ConfigError, parse_pipeline
from distributed_neural_networks_amd.models import build_golden_stage, default_ranges, kozusun, model_info
from distributed_neural_networks_amd.ops import decoder_ops as D_
from distributed_neural_networks_amd.runtime.engine import Engine, Entry
from distributed_neural_networks_amd.runtime.paging import PAGE, OutOfPages, PageTable, build_batch, pages_for
from distributed_neural_networks_amd.tools import trace_run


# ------------------------------------------------------------------ configuration
@pytest.mark.parametrize("name", sorted(CASES))
def test_config_and_tensor_names(name):
    d = CASES[name]
    c = kozusun.parse_config(d)
    n = c.n_layer
    assert [(r.layer, r.enters) for r in c.runs] == O.layer_runs(d)
    assert kozusun.stage_shapes(c, 0, n - 1, True, True) == O.tensor_shapes(d)
    # two stages together need every tensor
    cut = max(1, n // 2)
    parts = [kozusun.stage_shapes(c, 0, cut - 1, True, False), kozusun.stage_shapes(c, cut, n - 1, False, True)]
    assert set(parts[0]) | set(parts[1]) == set(O.tensor_shapes(d))
    assert "embed" in parts[0] and "head" in parts[1] and "head" not in parts[0]


def test_loop_order():
    c = kozusun.parse_config(config([layer(att(1, 1, 8, 8, 1.0))] * 5, 8, 8, loop=(1, 4, 2)))
    assert [(r.layer, r.enters) for r in c.runs] == [(0, False), (1, True), (2, False), (3, False), (1, True),
                                                     (2, False), (3, False), (4, False)]


@pytest.mark.parametrize("edit", [
    lambda d: d.update(architecture="Other"), lambda d: d.update(layers=[]), lambda d: d.pop("vocab"),
    lambda d: d["layers"][0].update(type="other"), lambda d: d["layers"][0]["mlp"].update(kind="other"),
    lambda d: d["layers"][0]["mixer"].update(kv_heads=3), lambda d: d["layers"][0]["mixer"].update(scale=-1.0),
    lambda d: d["layers"][0]["mixer"].pop("dim"), lambda d: d["layers"][0]["mixer"]["mask"].update(size=0),
    lambda d: d.update(loop={"start": 2, "stop": 9, "times": 2}), lambda d: d.pop("norm"),
])
def test_config_errors(edit):
    d = copy.deepcopy(CASES["plain"])
    edit(d)
    with pytest.raises(kozusun.ModelConfigError):
        kozusun.parse_config(d)


def test_model_folder(tmp_path):
    d = CASES["mixed"]
    W = O.random_weights(d, 1)
    O.save_model(str(tmp_path), d, W)
    info = model_info(str(tmp_path))
    assert info.family == "kozusun" and info.num_layers == len(O.layer_runs(d))
    assert len(default_ranges(str(tmp_path), 2)) == 2
    sd = ckpt.stage_state_dict(info.name, ckpt.load_full_state_dict(str(tmp_path)), 0, info.num_layers - 1, True, True)
    assert all(torch.equal(sd[k].float(), W[k]) for k in W)
    assert ckpt.unexpected_keys(info.name, sd, 0, 0, True, False)
    with pytest.raises(ValueError, match="GPU"):
        build_golden_stage(info.name, 0, info.num_layers - 1, True, True)
    bad = dict(sd)
    bad["l0.mix.q"] = bad["l0.mix.q"][:-1]
    with pytest.raises(ckpt.CheckpointError, match="l0.mix.q"):
        ckpt.stage_state_dict(info.name, bad, 0, info.num_layers - 1, True, True)
    del bad["l0.mix.q"]
    with pytest.raises(ckpt.CheckpointError, match="missing"):
        ckpt.stage_state_dict(info.name, bad, 0, info.num_layers - 1, True, True)
    pipe = {"nodes": [{"id": "n", "address": "127.0.0.1:5", "part_index": 0}], "model_weights": str(tmp_path),
            "num_parts": 1, "transport": "colocated", "model": str(tmp_path)}
    assert parse_pipeline(pipe).model == str(tmp_path)
    with pytest.raises(ConfigError, match="unknown model"):
        parse_pipeline(dict(pipe, model=str(tmp_path / "nothing")))
    other = tmp_path / "other"
    other.mkdir()
    (other / "config.json").write_text('{"architecture": "Other"}')
    with pytest.raises(KeyError, match="Other"):
        model_info(str(other))


def test_random_weights_are_stage_slices():
    n = model_info("kozusun-tiny").num_layers
    full = ckpt.random_stage_state_dict("kozusun-tiny", 0, n - 1, True, True, 3, nontrivial=True)
    part = ckpt.random_stage_state_dict("kozusun-tiny", 2, n - 1, False, True, 3, nontrivial=True)
    assert part and all(torch.equal(full[k], v) for k, v in part.items())


# ------------------------------------------------------------------ pages
def test_page_table_reuse():
    t = PageTable(6, 2)
    a, b = t.admit(), t.admit()
    with pytest.raises(OutOfPages):
        t.admit()
    t.reserve(a, PAGE)
    t.reserve(b, 1)
    t.reserve(a, PAGE + 1)
    assert t.table[a, :2].tolist() == [0, 2] and t.table[b, 0] == 1 and t.free_pages == 3
    t.reserve(a, 2 * PAGE)
    assert t.free_pages == 3
    with pytest.raises(OutOfPages):
        t.reserve(b, 5 * PAGE)
    assert t.free_pages == 3 and t.table[b, 1] == -1
    t.release(a)
    assert (t.table[a] == -1).all()
    c = t.admit()
    t.reserve(c, 3 * PAGE)
    assert c == a and set(t.table[c, :3].tolist()) >= {0, 2}  # freed pages come back first
    assert len(set(t.table[c, :3].tolist()) | {t.table[b, 0]}) == 4


def test_build_batch():
    t = PageTable(8, 3)
    s = [t.admit() for _ in range(3)]
    for x in s:
        t.reserve(x, 70)
    b = build_batch([([7, 8, 9], 64, s[0], [0, 2]), ([5], 3, s[1], []), (list(range(90)), 0, s[2], [89])], t.table,
                    [1, 3, 3], "cpu")
    assert b.M == 94 and b.n_dec == 1 and b.dec_rows.tolist() == [3] and b.want.tolist() == [0, 2, 93]
    assert b.pos[:5].tolist() == [64, 65, 66, 3, 0] and b.slots[[0, 3, 4]].tolist() == s
    assert b.chunks == [(0, 3, s[0]), (4, 90, s[2])] and b.max_len == 90
    assert b.tiles[1].tolist() == [[0, 3, s[0], 0], [4, 90, s[2], 0]]
    assert b.tiles[3].tolist() == [[0, 3, s[0], 0], [4, 90, s[2], 256], [4, 90, s[2], 128], [4, 90, s[2], 0]]
    assert torch.equal(b.table, torch.from_numpy(t.table))
    assert all(v.data_ptr() % 16 == b.ids.data_ptr() % 16 for v in b.tiles.values())
    with pytest.raises(ValueError):
        build_batch([([], 0, 0, [])], t.table, [1], "cpu")


def test_padding_rules():
    assert [D_.pad_dim(d) for d in (1, 64, 65, 128, 129, 256)] == [64, 64, 128, 128, 256, 256]
    with pytest.raises(ValueError):
        D_.pad_dim(257)
    assert D_.paged_splits(1, 8, 8, 4096, None, 0) > 1 and D_.paged_splits(1, 8, 8, 100, None, 0) == 1
    assert D_.paged_splits(1, 8, 8, 100000, 64, 8) == 1  # a short window needs no split


# ------------------------------------------------------------------ engine over a stand-in stage
class FakeStage:
    """Keeps the tokens of every sequence in pages; the next token is a hash of
    the whole sequence read back through the block table."""
    first = last = True
    model, V, groups = "fake", 50, [1]

    def __init__(self, num_pages, max_tokens):
        self.device, self.num_pages, self.max_tokens = torch.device("cpu"), num_pages, max_tokens
        self.pool = np.full((num_pages, PAGE), 1000)
        self.steps = []

    @staticmethod
    def next_token(seq):
        h = 7
        for t in seq:
            h = (h * 31 + int(t)) % 1009
        return h % 50

    def step_batch(self, b, x=None):
        self.steps.append(b.M)
        rows = list(zip(b.ids.tolist(), b.pos.tolist(), b.slots.tolist()))
        table = b.table.numpy()
        for t, p, s in rows:
            self.pool[table[s, p // PAGE], p % PAGE] = t
        if not b.n_want:
            return None
        out = torch.zeros(b.n_want, self.V)
        for i, w in enumerate(b.want.tolist()):
            _, p, s = rows[w]
            out[i, self.next_token([self.pool[table[s, j // PAGE], j % PAGE] for j in range(p + 1)])] = 1
        return out

    def sample(self, logits, pos):
        return logits.argmax(-1)


def _greedy(prompt, steps):
    seq = list(prompt)
    for _ in range(steps):
        seq.append(FakeStage.next_token(seq))
    return seq[len(prompt):]


@pytest.mark.parametrize("budget,pages,slots", [(0, 32, 8), (5, 32, 3), (2, 4, 8), (64, 3, 2), (1, 8, 4)])
def test_engine_generate_schedules(budget, pages, slots):
    g = torch.Generator().manual_seed(budget)
    prompts = [torch.randint(0, 50, (n,), generator=g).tolist() for n in (1, 70, 3, 64, 65, 20, 2)]
    st = FakeStage(pages, 200)
    eng = Engine([st], max_slots=slots)
    assert eng.generate(prompts, 9, budget) == [_greedy(p, 9) for p in prompts]
    assert max(st.steps) <= (budget or 200)
    assert eng.table.free_pages == pages and eng.table.free_slots == slots and not eng.live
    assert eng.generate(prompts[:2], 1, budget) == [_greedy(p, 1) for p in prompts[:2]]


def test_engine_step_checks():
    eng = Engine([FakeStage(2, 150)], max_slots=1)
    for e in (Entry("a", []), Entry("a", [50]), Entry("a", [-1]), Entry("a", [1], [1])):
        with pytest.raises(ValueError):
            eng.step([e])
    with pytest.raises(ValueError):
        eng.step([Entry("a", [1]), Entry("a", [2])])
    with pytest.raises(ValueError):
        eng.step([Entry("a", [1] * 151)])
    with pytest.raises(OutOfPages):
        eng.step([Entry("a", [1]), Entry("b", [1])])
    with pytest.raises(OutOfPages):
        eng.step([Entry("a", [1] * 129)])
    assert not eng.live and eng.table.free_pages == 2  # a refused step takes nothing
    assert eng.step([Entry("a", [1, 2])]) is None
    assert eng.step([]) is None
    with pytest.raises(OutOfPages):
        eng.step([Entry("a", [1] * 127)])
    assert eng.live["a"].length == 2
    eng.end("a")
    with pytest.raises(OutOfPages):
        eng.generate([[1] * 120], 9)


def test_trace_runner_protocol(tmp_path, capsys):
    eng = Engine([FakeStage(4, 128)], max_slots=4)
    lines = [json.dumps({"step": 0, "entries": [{"id": "a", "tokens": [1, 2, 3], "want": [0, 2]},
                                                {"id": "b", "tokens": [4], "want": []}], "end": []}), "\n",
             json.dumps({"step": 1, "entries": [{"id": "b", "tokens": [5, 6], "want": []}], "end": ["a"]}),
             json.dumps({"step": 2, "entries": [{"id": "b", "tokens": [7], "want": [0]}], "end": ["b"]})]
    trace_run.run(eng, io.StringIO("\n".join(lines)), str(tmp_path))
    assert capsys.readouterr().out.split("\n")[:3] == ["done 0", "done 1", "done 2"]
    a = np.fromfile(tmp_path / "0.f32", dtype="<f4").reshape(2, 50)
    assert a.argmax(1).tolist() == [FakeStage.next_token([1]), FakeStage.next_token([1, 2, 3])]
    assert not (tmp_path / "1.f32").exists()
    assert np.fromfile(tmp_path / "2.f32", dtype="<f4").argmax() == FakeStage.next_token([4, 5, 6, 7])
    assert not eng.live and eng.table.free_pages == 4


# ------------------------------------------------------------------ what the inputs reveal
def test_oracle_mask_edges():
    ok = O.visible(12, {"size": 3, "keep_first": 2})
    assert ok[9].nonzero().view(-1).tolist() == [0, 1, 7, 8, 9]
    assert ok[1].nonzero().view(-1).tolist() == [0, 1]
    assert O.visible(5, None)[4].all()


MISTAKES = {
    "window one longer": lambda d, W: d["layers"][0]["mixer"]["mask"].update(size=41),
    "window one shorter": lambda d, W: d["layers"][0]["mixer"]["mask"].update(size=39),
    "one kept key less": lambda d, W: d["layers"][0]["mixer"]["mask"].update(keep_first=4),
    "one kept key more": lambda d, W: d["layers"][0]["mixer"]["mask"].update(keep_first=6),
    "one pass less": lambda d, W: d["loop"].update(times=2),
    "residual multiplier": lambda d, W: d.update(residual_mult=1.0),
    "embedding scale": lambda d, W: d["embedding"].update(scale=3.3),
    "score scale": lambda d, W: d["layers"][2]["mixer"].update(scale=0.125),
    "loop sees the wrong half": lambda d, W: W.update({"loop.in": W["loop.in"].roll(128, 1)}),
    "no gate": lambda d, W: W.update({"l1.mix.g": W["l1.mix.g"] * 0}),
    "no key bias": lambda d, W: W.update({"l0.mix.q.b": W["l0.mix.q.b"] * 0}),
    "side part of another layer": lambda d, W: W.update({"side.embed": W["side.embed"].roll(16, 1)}),
    "plain final norm": lambda d, W: W.update({"final.norm": W["final.norm"] - 1}),
}


@pytest.mark.parametrize("name", sorted(MISTAKES))
def test_mistakes_show_in_logits(name):
    """A mistake planted in the oracle moves the logits by far more than the
    tolerance of the GPU comparison (2e-5): the random weights hide none."""
    d = copy.deepcopy(CASES["plain"])
    W = {k: v.double() for k, v in O.random_weights(d, 5, gain=1.5).items()}
    toks = torch.randint(0, d["vocab"], (90,), generator=torch.Generator().manual_seed(2))
    ref = O.forward(toks, d, W)
    MISTAKES[name](d, W)
    got = O.forward(toks, d, W)
    assert ((got - ref).norm() / ref.norm()).item() > 2e-3


def test_oracle_gelu():
    z = torch.linspace(-4, 4, 33, dtype=torch.float64)
    assert torch.allclose(O.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    assert math.isclose(O.rms_norm(torch.full((4,), 2.0, dtype=torch.float64), 0.0)[0].item(), 1.0)
