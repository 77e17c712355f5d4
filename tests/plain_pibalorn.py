"""Plain, slow implementations (numpy, float64) of the mechanisms of the Pibalorn design, one function per mechanism: the oracle of
tests/test_*pibalorn*.py, tests/test_gpu_gqa_ops.py and tests/test_gpu_linear_ops.py.  Nothing here is shared with powerinfer_amd/.

Weights are float arrays [out, in]; x rows are tokens.
"""
import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def unit(x, eps):
    """x over its root mean square (last axis)."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def layer_norm(x, w, eps):
    c = x - x.mean(axis=-1, keepdims=True)
    return c / np.sqrt(np.mean(c * c, axis=-1, keepdims=True) + eps) * w


def bigram_rows(tokens, previous, buckets, mul_prev, mul_cur):
    """Row of the bigram table of every token; previous: the token before the first one, None at the start of a sequence."""
    rows, p = [], previous
    for t in tokens:
        rows.append(buckets if p is None else (p * mul_prev + t * mul_cur) % buckets)
        p = t
    return rows


def embedding(tokens, previous, table, bigram, cfg):
    b = cfg["bigram"]
    return table[np.asarray(tokens)] * cfg["scale"] + bigram[bigram_rows(tokens, previous, b["buckets"], b["mul_prev"], b["mul_cur"])]


def rotate_halves(x, pos, dims, base):
    """Rotary embedding of the first `dims` of the last axis, element i paired with i + dims / 2; x [n_tok, heads, dim], pos [n_tok]."""
    h = dims // 2
    a = np.asarray(pos, np.float64)[:, None] * (float(base) ** (-2.0 * np.arange(h) / dims))[None, :]
    c, s = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    u, v = x[..., :h], x[..., h:dims]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., dims:]], axis=-1)


def softmax_plus_one(scores):
    """exp(s) / (1 + sum exp(s)) over the last axis; scores may contain -inf."""
    m = np.maximum(scores.max(axis=-1, keepdims=True), 0.0)
    e = np.exp(scores - m)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(-m))


def queries_and_cells(h, pos, t, m, eps):
    """(queries [n, H, dim], keys [n, G, dim], values [n, G, dim]) of the tokens h at positions pos."""
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    q, k = (h @ t["q"].T).reshape(-1, H, D), (h @ t["k"].T).reshape(-1, G, D)
    turn = lambda x: unit(rotate_halves(x, pos, m["rot"]["dims"], m["rot"]["base"]), eps)  # noqa: E731
    return turn(q), turn(k), k


def grouped_attention(q, keys, values, pos, kpos, scale):
    """[n, H, dim]: every query head against the keys of its group at positions not beyond its own."""
    n, H, D = q.shape
    per = H // keys.shape[1]
    seen = np.asarray(kpos)[None, :] <= np.asarray(pos)[:, None]
    out = np.empty((n, H, values.shape[2]))
    for a in range(H):
        s = np.where(seen, q[:, a] @ keys[:, a // per].T * scale, -np.inf)
        out[:, a] = softmax_plus_one(s) @ values[:, a // per]
    return out


def decayed_sums(q, k, v, decay, state):
    """Linear attention with a constant decay per head, token by token: q, k [n, H, dim], v [n, H, vdim], state [H, dim, vdim].
    Returns (outputs [n, H, vdim], state behind the last token)."""
    out, d = [], np.asarray(decay, np.float64)[:, None, None]
    for i in range(q.shape[0]):
        state = d * state + k[i][:, :, None] * v[i][:, None, :]
        out.append(np.einsum("hdv,hd->hv", state, q[i]))
    return np.asarray(out), state


def lightning(h, t, m, eps, state):
    """(mixer output [n, width], new state)."""
    n, H = h.shape[0], m["heads"]
    q, k, v = (silu(h @ t[x].T).reshape(n, H, -1) for x in "qkv")
    o, state = decayed_sums(q, k, v, m["decay"], state)
    return (unit(o.reshape(n, -1), eps) * t["norm"] * sigmoid(h @ t["g"].T)) @ t["o"].T, state


def clamped_glu(h, gate, up, down, limit):
    g = np.minimum(h @ gate.T, limit)
    u = np.clip(h @ up.T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def route_softmax(h, w_router, top):
    """(chosen experts [n, top] by falling logit, their weights).  route_softmax.margins: how far the closest decision was per token."""
    z = h @ w_router.T
    ids = np.argsort(-z, axis=1, kind="stable")
    by = np.take_along_axis(z, ids, 1)
    route_softmax.margins = by[:, top - 1] - by[:, top] if top < z.shape[1] else np.full(z.shape[0], np.inf)
    c = by[:, :top]
    e = np.exp(c - c.max(axis=1, keepdims=True))
    return ids[:, :top], e / e.sum(axis=1, keepdims=True)


def mixture(h, t, f):
    """t: router, experts [(gate, up, down)], shared (gate, up, down) or None, sg."""
    ids, w = route_softmax(h, t["router"], f["router"]["top"])
    out = np.zeros((h.shape[0], t["experts"][0][2].shape[0]))
    for i in range(h.shape[0]):
        for e, we in zip(ids[i], w[i]):
            out[i] += we * clamped_glu(h[i:i + 1], *t["experts"][e], f["expert"]["limit"])[0]
    if t["shared"] is not None:
        out += sigmoid(h @ t["sg"].T) * clamped_glu(h, *t["shared"], f["shared"]["limit"])
    return out


class PlainModel:
    """The whole decoder with the keys, values and states of every token seen so far; tensors: name -> float array."""

    def __init__(self, config, tensors):
        self.c, self.t = config, {k: np.asarray(v, np.float64) for k, v in tensors.items()}
        self.clear()

    def clear(self):
        self.kv, self.state = {}, {}
        self.n, self.previous = 0, None
        self.streams, self.margins = [], np.empty(0)       # margins: closest routing decision of every token so far

    def _mix(self, i, run, h, pos):
        ly, p, eps = self.c["layers"][i], f"l{i}.mix.", self.c["norm"]["eps"]
        m = ly["mixer"]
        if ly["type"] == "attention":
            q, k, v = queries_and_cells(h, pos, {x: self.t[p + x] for x in "qk"}, m, eps)
            old = self.kv.get(run)
            self.kv[run] = (k, v) if old is None else (np.concatenate([old[0], k]), np.concatenate([old[1], v]))
            k, v = self.kv[run]
            return grouped_attention(q, k, v, pos, np.arange(k.shape[0]), m["scale"]).reshape(h.shape[0], -1) @ self.t[p + "o"].T
        s = self.state.get(run, np.zeros((m["heads"], m["dim"], m["vdim"])))
        y, self.state[run] = lightning(h, {x: self.t[p + x] for x in ("q", "k", "v", "g", "o", "norm")}, m, eps, s)
        return y

    def _ff(self, i, h):
        f, p = self.c["layers"][i]["mlp"], f"l{i}.mlp."
        glu = lambda x: tuple(self.t[p + x + k] for k in ("gate", "up", "down"))  # noqa: E731
        if f["kind"] == "dense":
            return clamped_glu(h, *glu(""), f["limit"])
        return mixture(h, {"router": self.t[p + "router"], "experts": [glu(f"e{e}.") for e in range(f["router"]["experts"])],
                           "shared": glu("shared.") if f.get("shared") else None, "sg": self.t.get(p + "shared.sg")}, f)

    def order(self):
        """(layer, pass number if a pass starts with it, else None) of every layer run."""
        lo, n = self.c.get("loop"), len(self.c["layers"])
        if not lo:
            return [(i, None) for i in range(n)]
        loop = [(i, t if i == lo["start"] else None) for t in range(lo["times"]) for i in range(lo["start"], lo["stop"])]
        return [(i, None) for i in range(lo["start"])] + loop + [(i, None) for i in range(lo["stop"], n)]

    def feed(self, tokens):
        """Logits [n, vocab] of the next tokens of the sequence; self.streams: the residual stream after every layer run."""
        eps, t = self.c["norm"]["eps"], self.t
        tokens = [int(v) for v in tokens]
        pos = np.arange(self.n, self.n + len(tokens))
        x0 = embedding(tokens, self.previous, t["embed"], t["bigram"], self.c["embedding"])
        self.n, self.previous = self.n + len(tokens), tokens[-1]
        self.streams, margins, x = [], np.full(len(tokens), np.inf), x0
        for run, (i, start) in enumerate(self.order()):
            if start is not None:
                x = x + (x0 if start else 0.0) + t["loop.step"][start]
            h = layer_norm(x, t[f"l{i}.norm1"], eps)
            y = self._mix(i, run, h, pos)
            f = self.c["layers"][i]["mlp"]
            if f is not None:
                y = y + self._ff(i, h)
                if f["kind"] == "moe":
                    margins = np.minimum(margins, route_softmax.margins)
            x = x + y
            self.streams.append(x)
        self.margins = np.concatenate([self.margins, margins])
        return layer_norm(x, t["final.norm"], eps) @ t["head"].T
