"""Plain, slow implementations (numpy, float64) of the mechanisms of the Pufivik design, one function per mechanism: the oracle of
tests/test_*pufivik*.py and of the operator tests of its kernels.  Nothing here is shared with powerinfer_amd/.

Weights are float arrays [out, in]; x rows are tokens.
"""
import math

import numpy as np


def sigmoid(z):
    return np.where(z >= 0, 1.0, np.exp(-np.abs(z))) / (1.0 + np.exp(-np.abs(z)))


def silu(z):
    return z * sigmoid(z)


def embedding(tokens, table, scale):
    return table[np.asarray(tokens)] * scale


# ---- norms, residual, convolution over time -----------------------------------------------------------------------------------------
def group_norm(x, w, groups, eps):
    """Every one of `groups` equal parts of the last axis over its own root mean square, the whole times w."""
    parts = x.reshape(*x.shape[:-1], groups, -1)
    return (parts / np.sqrt(np.mean(parts * parts, axis=-1, keepdims=True) + eps)).reshape(x.shape) * w


def add_normed(x, y, mult, w, groups, eps):
    """The residual stream behind a sublayer with the result y."""
    return x + mult * group_norm(y, w, groups, eps)


def past_inputs(past, h, taps):
    """The last taps - 1 inputs once h has been read."""
    both = np.concatenate([past, h])
    return both[both.shape[0] - (taps - 1):]


def convolved(h, past, w):
    """h plus its causal convolution over time, channel by channel; w [width, taps], the last tap at the token itself; past [taps - 1, width]."""
    taps, n = w.shape[1], h.shape[0]
    rows = np.concatenate([past, h])
    return h + sum(w[:, j] * rows[j:j + n] for j in range(taps))


# ---- rotations ----------------------------------------------------------------------------------------------------------------------
def plain_frequencies(dims, base):
    return float(base) ** (-2.0 * np.arange(dims // 2) / dims) if dims else np.empty(0)


def wavelength_frequencies(dims, base, s):
    """Frequencies of long waves divided by a factor, those in between blended by how often the wave fits into the original context."""
    out = []
    for f in plain_frequencies(dims, base):
        turns = s["original"] * f / (2 * math.pi)
        if turns > s["high"]:
            out.append(f)
        elif turns < s["low"]:
            out.append(f / s["factor"])
        else:
            a = (turns - s["low"]) / (s["high"] - s["low"])
            out.append((1 - a) * f / s["factor"] + a * f)
    return np.asarray(out)


def ramp_frequencies(dims, base, s):
    """Frequencies blended between kept and divided by a factor along a ramp over the dimensions."""
    at = lambda turns: dims * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))  # noqa: E731
    lo, hi = max(math.floor(at(s["fast"])), 0), min(math.ceil(at(s["slow"])), dims - 1)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0, 1)
    f = plain_frequencies(dims, base)
    return f / s["factor"] * ramp + f * (1 - ramp)


def ramp_length(s):
    """What the ramp's rotation multiplies the rotated part by."""
    return 0.1 * math.log(s["factor"]) + 1


def rotate_halves(x, pos, f, length=1.0):
    """Element i of the first 2 len(f) paired with element i + len(f); x [n_tok, heads, dim], pos [n_tok]."""
    a, h = np.asarray(pos, np.float64)[:, None] * f[None, :], len(f)
    c, s = length * np.cos(a)[:, None, :], length * np.sin(a)[:, None, :]
    u, v = x[..., :h], x[..., h:2 * h]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., 2 * h:]], axis=-1)


def rotate_neighbours(x, pos, f, length=1.0):
    """Element 2 i paired with 2 i + 1."""
    a, n = np.asarray(pos, np.float64)[:, None] * f[None, :], 2 * len(f)
    c, s = length * np.cos(a)[:, None, :], length * np.sin(a)[:, None, :]
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    y = np.array(x)
    y[..., 0:n:2], y[..., 1:n:2] = u * c - v * s, v * c + u * s
    return y


# ---- attention ----------------------------------------------------------------------------------------------------------------------
def blended_values(v, first, lam):
    return (1 - lam) * v + lam * first


def scores(q, keys, scale):
    """[H, n, keys]: every query head against the keys of its group."""
    per = q.shape[1] // keys.shape[1]
    return np.stack([q[:, a] @ keys[:, a // per].T for a in range(q.shape[1])]) * scale


def capped(s, cap):
    return cap * np.tanh(s / cap)


def causal(s, pos, kpos):
    return np.where(np.asarray(kpos)[None, :] <= np.asarray(pos)[:, None], s, -np.inf)


def softmax(s, sink=None):
    """Along the last axis of s [H, n, keys]; sink [H]: one more entry of the denominator."""
    m = s.max(axis=-1, keepdims=True)
    if sink is not None:
        m = np.maximum(m, sink[:, None, None])
    e = np.exp(s - m)
    den = e.sum(axis=-1, keepdims=True)
    if sink is not None:
        den = den + np.exp(sink[:, None, None] - m)
    return e / den


def mixed_heads(w, talk):
    """Weights [H, n, keys], each head's a mixture of all heads'."""
    return np.einsum("hg,gnk->hnk", talk, w)


def weighted_values(w, values):
    """[n, H, vdim]: every head's weights on the values of its group."""
    per = w.shape[0] // values.shape[1]
    return np.stack([w[a] @ values[:, a // per] for a in range(w.shape[0])], axis=1)


def gated_heads(o, h, g):
    """[n, H, vdim], every head times a number of its token."""
    return o * sigmoid(h @ g.T)[:, :, None]


# ---- experts ------------------------------------------------------------------------------------------------------------------------
def choice(h, router, top):
    """(experts [n, top] by falling score, their scores)."""
    s = sigmoid(h @ router.T)
    ids = np.argsort(-s, axis=1, kind="stable")[:, :top]
    return ids, np.take_along_axis(s, ids, 1)


def expert(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def experts(h, t, top):
    """t: router and e<k>.gate, .up, .down; a chosen expert reads the token times its score."""
    ids, w = choice(h, t["router"], top)
    out = np.zeros_like(h)
    for i in range(h.shape[0]):
        for e, f in zip(ids[i], w[i]):
            out[i] += expert((f * h[i])[None], t[f"e{e}.gate"], t[f"e{e}.up"], t[f"e{e}.down"])[0]
    return out


class PlainModel:
    """The whole decoder with the keys, values and convolution inputs of every token seen so far; tensors: name -> float array."""

    def __init__(self, config, tensors):
        self.c, self.t = config, {k: np.asarray(v, np.float64) for k, v in tensors.items()}
        self.clear()

    def clear(self):
        self.kv, self.past = {}, {}
        self.n, self.streams = 0, []

    def sub(self, prefix):
        return {k[len(prefix):]: v for k, v in self.t.items() if k.startswith(prefix)}

    def turn(self, kind, x, pos, rot):
        if not rot:
            return x
        s = rot.get("scaling")
        if kind == "attention":
            return rotate_halves(x, pos, wavelength_frequencies(rot["dims"], rot["base"], s) if s else plain_frequencies(rot["dims"], rot["base"]))
        if not s:
            return rotate_neighbours(x, pos, plain_frequencies(rot["dims"], rot["base"]))
        return rotate_neighbours(x, pos, ramp_frequencies(rot["dims"], rot["base"], s), ramp_length(s))

    def attend(self, i, h, pos):
        kind, m = self.c["layers"][i]["type"], self.c["layers"][i]["mixer"]
        t, n = self.sub(f"l{i}.mix."), h.shape[0]
        q, k, v = ((h @ t[x].T).reshape(n, heads, -1) for x, heads in (("q", m["heads"]), ("k", m["kv_heads"]), ("v", m["kv_heads"])))
        if m.get("v_mix"):
            if self.first_values is None:
                self.first_values = v
            else:
                v = blended_values(v, self.first_values, t["vmix"])
        q, k = self.turn(kind, q, pos, m["rot"]), self.turn(kind, k, pos, m["rot"])
        old = self.kv.get(i)
        self.kv[i] = (k, v) if old is None else (np.concatenate([old[0], k]), np.concatenate([old[1], v]))
        k, v = self.kv[i]
        s = scores(q, k, m["scale"])
        if kind == "attention_2":
            s = capped(s, m["softcap"])
        s = causal(s, pos, np.arange(k.shape[0]))
        if kind == "attention_2":
            o = weighted_values(softmax(s), v)
        else:
            o = gated_heads(weighted_values(mixed_heads(softmax(s, t["sink"]), t["talk"]), v), h, t["g"])
        return o.reshape(n, -1) @ t["o"].T

    def operand(self, x):
        """What a sublayer reads of its norm's result."""
        return x

    def feed(self, tokens):
        """Logits [n, vocab] of the next tokens of the sequence; self.streams: the residual stream after every layer."""
        t, mult, taps = self.t, self.c["residual_mult"], self.c["canon"]["taps"]
        norm = self.c["norm"]["groups"], self.c["norm"]["eps"]
        tokens = [int(v) for v in tokens]
        pos = np.arange(self.n, self.n + len(tokens))
        self.n += len(tokens)
        x = embedding(tokens, t["embed"], self.c["embedding"]["scale"])
        self.streams, self.first_values = [], None
        for i, ly in enumerate(self.c["layers"]):
            p = f"l{i}."
            h = group_norm(x, t[p + "norm1"], *norm)
            past = self.past.get(i, np.zeros((taps - 1, x.shape[1])))
            self.past[i] = past_inputs(past, h, taps)
            h = self.operand(convolved(h, past, t[p + "canon1"]))
            x = add_normed(x, self.attend(i, h, pos), mult, t[p + "norm1b"], *norm)
            if ly["mlp"] is not None:
                h = self.operand(group_norm(x, t[p + "norm2"], *norm))
                x = add_normed(x, experts(h, self.sub(p + "mlp."), ly["mlp"]["router"]["top"]), mult, t[p + "norm2b"], *norm)
            self.streams.append(x)
        return group_norm(x, t["final.norm"], *norm) @ t["embed"].T
