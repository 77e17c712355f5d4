"""Host-side parts of the Lerasun path (no GPU): checkpoint files, configuration, scheduling, and the oracle itself - that its answers do
not depend on how a prompt is cut, and that it tells a mistake in any mechanism from rounding."""
import json
import os

import numpy as np
import pytest

import plain_latent as pl_oracle
from lerasun_models import config, even_config, layer, odd_config, row_errors, tokens, weights
from powerinfer_amd import checkpoint, lerasun, registry, serve


def test_safetensors_round_trip(tmp_path):
    rng = np.random.default_rng(0)
    t = {"a": checkpoint.bf16_bits(rng.standard_normal((3, 5))), "b": rng.standard_normal(7).astype(np.float32), "c": np.arange(6, dtype=np.int32).reshape(2, 3)}
    checkpoint.write_safetensors(tmp_path / "m.safetensors", t)
    back = checkpoint.read_safetensors(tmp_path / "m.safetensors")
    assert set(back) == set(t)
    for k in t:
        assert back[k].dtype == t[k].dtype and np.array_equal(back[k], t[k])


def test_safetensors_refuses_broken_files(tmp_path):
    p = tmp_path / "m.safetensors"
    p.write_bytes(b"\xff" * 16)
    with pytest.raises(ValueError):
        checkpoint.read_safetensors(p)
    checkpoint.write_safetensors(p, {"a": np.zeros(4, np.float32)})
    p.write_bytes(p.read_bytes()[:-4])
    with pytest.raises(ValueError):
        checkpoint.read_safetensors(p)


def test_bf16_rounding_is_to_nearest_even():
    x = np.array([1.0, 1.00390625, 1.01171875, -2.5, 3.0e38, 1e-40], np.float32)      # ties go to the even pattern
    import torch
    want = torch.tensor(x).to(torch.bfloat16).view(torch.int16).numpy().view(np.uint16)
    assert np.array_equal(checkpoint.bf16_bits(x), want)
    assert np.array_equal(checkpoint.bf16_floats(want), torch.tensor(x).to(torch.bfloat16).float().numpy())


def test_descriptions_follow_the_configuration():
    d = lerasun.layer_descs(odd_config())
    assert [x["kv_from"] for x in d] == [-1, 0, -1, 2, 0] and d[1]["ffn"] == 0 and d[2]["n_group"] == 1 and d[3]["rot_base"] == 500.0
    assert (d[0]["n_expert"], d[0]["n_top"], d[0]["n_group"], d[0]["n_group_keep"], d[0]["expert_ff"]) == (6, 2, 3, 2, 24)
    c = odd_config()
    c["layers"][0]["type"] = "something_else"
    with pytest.raises(ValueError):
        lerasun.layer_descs(c)
    c = odd_config()
    c["layers"][0]["mlp"]["kind"] = "dense"
    with pytest.raises(ValueError):
        lerasun.layer_descs(c)
    c = odd_config()
    del c["layers"][0]["mlp"]["router"]["groups"]
    assert lerasun.layer_descs(c)[0]["n_group"] == 1


def test_registry_refuses_unknown_designs(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "NoSuchDesign"}))
    with pytest.raises(ValueError, match="not registered"):
        registry.load_model(str(tmp_path))
    assert "Lerasun" in registry.FOLDERS


class FakeModel:
    """Counts cells as the engine does and answers (last token + position + 1) % 97 as the next token."""

    def __init__(self):
        self.hp = type("HP", (), {"n_vocab": 97})
        self.cells, self.n_cells, self.peak, self.batches = {}, 0, 0, []

    def kv_cells_init(self, n):
        self.n_cells = n

    def kv_cells_step(self, tokens, positions, masks, want, want_logits=True, want_next=True):
        for t, p, m in zip(tokens, positions, masks):
            assert len(self.cells.setdefault(m, [])) == p, "positions of a sequence follow one another"
            self.cells[m].append(t)
        used = sum(map(len, self.cells.values()))
        assert used <= self.n_cells
        self.peak = max(self.peak, used)
        self.batches.append(len(tokens))
        nxt = np.array([(tokens[w] + positions[w] + 1) % 97 for w in want], np.int32)
        return nxt, None

    def kv_cells_seq_rm(self, s, p0, p1):
        self.cells.pop(1 << s, None)


def expected(prompt, n):
    out, pos = [], len(prompt) - 1
    t = prompt[-1]
    for _ in range(n):
        t = (t + pos + 1) % 97
        out.append(t)
        pos += 1
    return out


@pytest.mark.parametrize("budget,cells,live", [(7, 64, 3), (512, 200, 16), (1, 40, 2)])
def test_scheduler_keeps_within_the_pool_and_finishes_everything(budget, cells, live):
    m = FakeModel()
    s = serve.Scheduler(m, cells, max_live=live, budget=budget)
    rng = np.random.default_rng(4)
    want = {}
    for i in range(12):
        p, n = [int(v) for v in rng.integers(0, 97, rng.integers(1, 20))], int(rng.integers(1, 12))
        s.submit(i, p, n)
        want[i] = expected(p, n)
    assert s.run() == want
    assert not m.cells and m.peak <= cells and max(m.batches) <= max(budget, live)


def test_scheduler_stops_at_the_end_token_and_refuses_what_cannot_fit():
    m = FakeModel()
    s = serve.Scheduler(m, 32)
    full = expected([5, 6], 20)
    s.submit("x", [5, 6], 20, eos=full[3])
    with pytest.raises(ValueError):
        s.submit("y", [1] * 30, 10)
    with pytest.raises(ValueError):
        s.submit("z", [], 4)
    assert s.run()["x"] == full[:full.index(full[3]) + 1]


def test_stepper_hands_sequences_out_again():
    st = serve.Stepper(FakeModel(), 64, max_live=2)
    st.run([("a", [1, 2], [1]), ("b", [3], [0])], logits=False, greedy=True)
    with pytest.raises(RuntimeError):
        st.run([("c", [4], [0])], logits=False, greedy=True)
    st.end("a")
    _, nxt = st.run([("c", [4], [0]), ("b", [9], [])], logits=False, greedy=True)
    assert nxt.tolist() == [5] and st.free_cells == 64 - 1 - 2


# ---- the oracle ----------------------------------------------------------------------------------------------------------------
def test_oracle_does_not_depend_on_the_cut():
    cfg = odd_config()
    m = pl_oracle.PlainModel(cfg, weights(cfg, 1))
    toks = tokens(cfg, 40, 2)
    whole = m.feed(toks)
    m.clear()
    parts = []
    for a, b in zip([0, 2, 3, 19, 20], [2, 3, 19, 20, 40]):
        parts.append(m.feed(toks[a:b]))
    assert np.abs(np.vstack(parts) - whole).max() < 1e-10


def planted(name):
    """(patched attribute, faulty function)"""
    o = pl_oracle
    soft = o.sink_softmax
    return {
        "no sink": ("sink_softmax", lambda s, k: soft(s, np.full_like(k, -1e9))),
        "sink counted twice": ("sink_softmax", lambda s, k: soft(s, k + np.log(2.0))),
        "rotation of halves": ("rotate_pairs", lambda x, p, b: np.concatenate(
            [x[..., :x.shape[-1] // 2], x[..., x.shape[-1] // 2:]], -1)),
        "norm weight without its offset": ("rms_norm_zero", lambda x, w, e: o.rms(x, e) * w),
        "weights from choice scores": ("route", _route_weights_from_choice),
        "groups ignored": ("route", lambda h, w, c, t, g, k: _route(h, w, c, t, 1, 1)),
    }[name]


_route = pl_oracle.route


def _route_weights_from_choice(h, w, c, top, g, keep):
    ids, wt = _route(h, w, c, top, g, keep)
    s = 1 / (1 + np.exp(-(h @ w.T))) + c
    v = np.take_along_axis(s, ids, 1)
    return ids, v / v.sum(1, keepdims=True)


@pytest.mark.parametrize("name", ["no sink", "sink counted twice", "rotation of halves", "norm weight without its offset", "weights from choice scores", "groups ignored"])
def test_a_mistake_in_a_mechanism_shows(monkeypatch, name):
    cfg = even_config()
    w = weights(cfg, 3)
    toks = tokens(cfg, 48, 4)
    good = pl_oracle.PlainModel(cfg, w).feed(toks)
    attr, fn = planted(name)
    monkeypatch.setattr(pl_oracle, attr, fn)
    bad = pl_oracle.PlainModel(cfg, w).feed(toks)
    assert np.quantile(row_errors(bad, good), 0.75) > 0.05          # the model tests allow 0.02 in bf16, 2e-5 in fp32


def test_choice_scores_may_be_negative():
    """A closed group's experts count as minus infinity, not as zero: with negative choice scores everywhere they must not win."""
    h = np.zeros((1, 4))
    ids, wts = pl_oracle.route(h, np.zeros((6, 4)), np.array([-3.0, -3.1, -1.0, -5.0, -2.0, -2.1]), 2, 3, 1)
    assert ids[0].tolist() == [4, 5] and np.allclose(wts, 0.5)      # (sums with 0.5 added to each score: -5.1, -5.0, -3.1)


def test_entry_points_exist():
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    assert os.access(os.path.join(root, "bin", "trace_run"), os.X_OK)
    import powerinfer_amd.__main__ as cli
    with pytest.raises(SystemExit):
        cli.main(["generate"])
    assert config(8, 8, [layer(1, 2, 2, 2, 2)])["layers"][0]["mlp"] is None
