"""Host-side parts of the Pibalorn path (no GPU): configuration, registry, and the oracle itself - that its answers do not depend on how a
prompt is cut, and that it tells a mistake in any mechanism from rounding."""
import numpy as np
import pytest

import plain_pibalorn as o
from lerasun_models import row_errors, tokens
from pibalorn_models import attention, config, even_config, lightning, moe, odd_config, tall_config, weights
from powerinfer_amd import lib as pl, pibalorn, registry


def test_descriptions_follow_the_configuration():
    d = pibalorn.layer_descs(odd_config())
    assert [x["mixer"] for x in d] == [pl.MIXER_LINEAR, pl.MIXER_GROUPED, pl.MIXER_GROUPED, pl.MIXER_LINEAR, pl.MIXER_GROUPED]
    assert [x["ffn"] for x in d] == [pl.FFN_GLU_MOE, pl.FFN_GLU, pl.FFN_NONE, pl.FFN_GLU, pl.FFN_GLU_MOE]
    assert (d[1]["rot_dim"], d[1]["rot_base"], d[1]["n_kv_head"], d[1]["glu_ff"], d[1]["glu_limit"]) == (24, 500.0, 2, 90, 0.9)
    assert "glu_ff" not in d[0] and (d[0]["n_expert"], d[0]["n_top"], d[0]["expert_ff"], d[0]["expert_limit"]) == (7, 3, 23, 0.7)
    assert (d[4]["glu_ff"], d[4]["glu_limit"]) == (31, 0.8)
    assert pibalorn.model_opts(odd_config()) == dict(embed_scale=2.5, bigram_buckets=41, bigram_mul_prev=5, bigram_mul_cur=1000003, loop_start=0, loop_stop=1, loop_times=3)
    c = odd_config()
    del c["loop"], c["embedding"]["bigram"]
    assert pibalorn.model_opts(c) == dict(embed_scale=2.5)
    assert "Pibalorn" in registry.FOLDERS


@pytest.mark.parametrize("spoil", [lambda c: c["layers"][0].update(type="something"), lambda c: c["layers"][1]["mlp"].update(kind="other"),
                                   lambda c: c["layers"][2]["mixer"].update(vdim=5), lambda c: c["layers"][0]["mixer"]["decay"].pop()])
def test_what_the_design_does_not_have_is_refused(spoil):
    c = odd_config()
    spoil(c)
    with pytest.raises(ValueError, match="layer"):
        pibalorn.layer_descs(c)


@pytest.mark.parametrize("make", [odd_config, even_config, tall_config])
def test_oracle_does_not_depend_on_the_cut(make):
    cfg = make()
    m = o.PlainModel(cfg, weights(cfg, 1))
    toks = tokens(cfg, 40, 2)
    whole = m.feed(toks)
    assert len(m.streams) == len(m.order())
    m.clear()
    parts = [m.feed(toks[a:b]) for a, b in zip([0, 2, 3, 19, 20], [2, 3, 19, 20, 40])]
    assert np.abs(np.vstack(parts) - whole).max() < 1e-9


def test_layer_order_of_a_loop():
    cfg = config(8, 8, [lightning(1, 2, 2, [0.5])] * 4, loop=(1, 3, 2))
    assert o.PlainModel(cfg, {}).order() == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    cfg["loop"]["times"] = 1
    assert o.PlainModel(cfg, {}).order() == [(0, None), (1, 0), (2, None), (3, None)]


soft, rot, unit, bigram, glu, sums, soft_route = o.softmax_plus_one, o.rotate_halves, o.unit, o.bigram_rows, o.clamped_glu, o.decayed_sums, o.route_softmax


def neighbours(x, pos, dims, base):
    a = np.asarray(pos, np.float64)[:, None] * (float(base) ** (-2.0 * np.arange(dims // 2) / dims))[None, :]
    c, s = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    y = np.array(x)
    y[..., 0:dims:2], y[..., 1:dims:2] = x[..., 0:dims:2] * c - x[..., 1:dims:2] * s, x[..., 1:dims:2] * c + x[..., 0:dims:2] * s
    return y


def softmax(s):
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def values_after_norm(h, pos, t, m, eps):
    q, k, _ = queries(h, pos, t, m, eps)
    return q, k, k


def norm_first(h, pos, t, m, eps):
    q, k, v = queries(h, pos, t, m, eps)
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    return rot((h @ t["q"].T).reshape(-1, H, D), pos, m["rot"]["dims"], m["rot"]["base"]), rot((h @ t["k"].T).reshape(-1, G, D), pos, m["rot"]["dims"], m["rot"]["base"]), v


def whole_softmax(h, w, top):
    z = h @ w.T
    ids, _ = soft_route(h, w, top)
    return ids, np.take_along_axis(softmax(z), ids, 1)


def late_decay(q, k, v, decay, state):
    out, d = [], np.asarray(decay)[:, None, None]
    for i in range(q.shape[0]):
        state = d * (state + k[i][:, :, None] * v[i][:, None, :])
        out.append(np.einsum("hdv,hd->hv", state, q[i]))
    return np.asarray(out), state


queries = o.queries_and_cells
PLANTED = {
    "no added one": ("softmax_plus_one", softmax),
    "rotation of neighbours": ("rotate_halves", neighbours),
    "values behind norm and rotation": ("queries_and_cells", values_after_norm),
    "queries and keys not divided": ("queries_and_cells", norm_first),
    "rms instead of layer norm": ("layer_norm", lambda x, w, e: unit(x, e) * w),
    "first token hashed with zero": ("bigram_rows", lambda t, p, *a: bigram(t, 0 if p is None else p, *a)),
    "bigram factors swapped": ("bigram_rows", lambda t, p, b, mp, mc: bigram(t, p, b, mc, mp)),
    "gate clamped on both sides": ("clamped_glu", lambda h, g, u, d, limit: (lambda a: (a * o.sigmoid(1.702 * a) * (np.clip(h @ u.T, -limit, limit) + 1)) @ d.T)(np.clip(h @ g.T, -limit, limit))),
    "up without its one": ("clamped_glu", lambda h, g, u, d, limit: glu(h, g, u, d, limit) - (np.minimum(h @ g.T, limit) * o.sigmoid(1.702 * np.minimum(h @ g.T, limit))) @ d.T),
    "plain silu in the GLU": ("clamped_glu", lambda h, g, u, d, limit: (o.silu(np.minimum(h @ g.T, limit)) * (np.clip(h @ u.T, -limit, limit) + 1)) @ d.T),
    "no limits": ("clamped_glu", lambda h, g, u, d, limit: glu(h, g, u, d, 1e9)),
    "decay applied to the new pair": ("decayed_sums", late_decay),
    "state lost between calls": ("decayed_sums", lambda q, k, v, d, s: sums(q, k, v, d, s * 0)),
    "weights from all experts": ("route_softmax", whole_softmax),
}


@pytest.mark.parametrize("name", PLANTED)
def test_a_mistake_in_a_mechanism_shows(monkeypatch, name):
    cfg = even_config()
    w = weights(cfg, 3)
    toks = tokens(cfg, 48, 4)

    def run():
        m = o.PlainModel(cfg, w)
        return np.vstack([m.feed(toks[:20]), m.feed(toks[20:])])

    good = run()
    attr, fn = PLANTED[name]
    monkeypatch.setattr(o, attr, fn)
    e = row_errors(run(), good)
    if "first token" in name:
        assert e[0] > 0.05
    elif "decay" in name:                                   # a factor per head, which the norm behind the heads takes out in part
        assert np.median(e) > 5e-3
    elif "lost" in name:
        assert (e[:20] == 0).all() and e[20:].max() > 0.1
    else:
        assert np.quantile(e, 0.75) > 0.04              # the model tests allow 0.02 in bf16, 2e-5 in fp32


@pytest.mark.parametrize("what", ["loop step left out", "embedding not added again", "passes share a cache"])
def test_a_mistake_in_the_loop_shows(what):
    cfg = even_config()
    w = weights(cfg, 5)
    toks = tokens(cfg, 30, 6)
    good = o.PlainModel(cfg, w).feed(toks)
    m = o.PlainModel(cfg, w)
    if what == "loop step left out":
        m.t["loop.step"] = m.t["loop.step"] * [[1.0], [0.0]]
    elif what == "embedding not added again":
        order = m.order()
        m.order = lambda: [(i, None) if s else (i, s) for i, s in order]
    else:
        mix = m._mix
        m._mix = lambda i, run, h, pos: mix(i, i, h, pos)
    try:
        bad = m.feed(toks)
    except ValueError:                                  # (twice the keys do not fit the positions)
        return
    assert np.quantile(row_errors(bad, good), 0.75) > 0.04


def test_ties_and_single_experts():
    h, w = np.ones((1, 2)), np.array([[1.0, 0.0], [2.0, 0.0], [2.0, 0.0]])
    ids, wt = o.route_softmax(h, w, 2)
    assert ids[0].tolist() == [1, 2] and np.allclose(wt, 0.5)
    ids, wt = o.route_softmax(h, w, 1)
    assert ids[0].tolist() == [1] and wt[0, 0] == 1.0
    assert moe(3, 1, 4)["router"]["top"] == 1 and attention(2, 1, 4)["mixer"]["vdim"] == 4
