"""Plain, slow implementations (numpy, float64) of the mechanisms of the Fikevik design, one function per mechanism: the oracle of
tests/test_*fikevik*.py and of the operator tests of its kernels.  Nothing here is shared with powerinfer_amd/.

Weights are float arrays [out, in]; x rows are tokens.
"""
import numpy as np


def sigmoid(z):
    return np.where(z >= 0, 1.0, np.exp(-np.abs(z))) / (1.0 + np.exp(-np.abs(z)))


def log_sigmoid(z):
    return np.minimum(z, 0.0) - np.log1p(np.exp(-np.abs(z)))


def silu(z):
    return z * sigmoid(z)


def unit(x, eps):
    """x over its root mean square (last axis)."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return unit(x, eps) * w


def embedding(tokens, table, scale):
    return table[np.asarray(tokens)] * scale


def gated(y, h, w, b):
    """A sublayer's result times the gate its input opens."""
    return y * sigmoid(h @ w.T + b)


def norm_after_sum(x, y, alpha, w, eps):
    return rms_norm(alpha * x + y, w, eps)


def swiglu(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


# ---- grouped-query attention in a window --------------------------------------------------------------------------------------------
def rotate_neighbours(x, pos, dims, base):
    """Rotary embedding of the first `dims` of the last axis, element 2 i paired with 2 i + 1; x [n_tok, heads, dim], pos [n_tok]."""
    a = np.asarray(pos, np.float64)[:, None] * (float(base) ** (-2.0 * np.arange(dims // 2) / dims if dims else np.empty(0)))[None, :]
    c, s = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    y = np.array(x)
    y[..., 0:dims:2], y[..., 1:dims:2] = u * c - v * s, v * c + u * s
    return y


def head_norm(x, w, eps):
    """RMS norm of every head's vector, one weight for all heads."""
    return rms_norm(x, w, eps)


def head_scale(temp, scale):
    """What each query head's scores are multiplied by."""
    return scale * np.asarray(temp)


def in_window(pos, kpos, size):
    d = np.asarray(pos)[:, None] - np.asarray(kpos)[None, :]
    return (d >= 0) & (d < size)


def softmax(scores):
    e = np.exp(scores - scores.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def queries_and_cells(h, pos, t, m, eps):
    """(queries [n, H, dim], keys [n, G, dim], values [n, G, vdim]) of the tokens h at positions pos."""
    n, H, G = h.shape[0], m["heads"], m["kv_heads"]
    turn = lambda x: rotate_neighbours(x, pos, m["rot"]["dims"], m["rot"]["base"])  # noqa: E731
    q = head_norm((h @ t["q"].T).reshape(n, H, m["dim"]), t["q.norm"], eps)
    k = head_norm((h @ t["k"].T).reshape(n, G, m["dim"]), t["k.norm"], eps)
    return turn(q), turn(k), unit((h @ t["v"].T).reshape(n, G, m["vdim"]), eps)


def window_attention(q, keys, values, pos, kpos, scales, size):
    """[n, H, vdim]: every query head against the keys of its group inside the window; scales: one factor per query head."""
    n, H, _ = q.shape
    per = H // keys.shape[1]
    seen = in_window(pos, kpos, size)
    out = np.empty((n, H, values.shape[2]))
    for a in range(H):
        s = np.where(seen, q[:, a] @ keys[:, a // per].T * scales[a], -np.inf)
        out[:, a] = softmax(s) @ values[:, a // per]
    return out


# ---- gated linear attention: a decay per key channel and token ----------------------------------------------------------------------
def key_decays(h, a1, a2, b, tau):
    return np.exp(log_sigmoid((h @ a1.T) @ a2.T + b) / tau)


def keyed_sums(q, k, v, decay, state):
    """q, k, decay [n, H, dim], v [n, H, vdim], state [H, dim, vdim].  Returns (outputs [n, H, vdim], state behind the last token)."""
    out = []
    for i in range(q.shape[0]):
        state = decay[i][:, :, None] * state + k[i][:, :, None] * v[i][:, None, :]
        out.append(np.einsum("hdv,hd->hv", state, q[i]))
    return np.asarray(out).reshape(q.shape[0], *v.shape[1:]), state


def gla(h, t, m, eps, state):
    """(mixer output [n, width], new state)."""
    n, H = h.shape[0], m["heads"]
    q, k, v = ((h @ t[x].T).reshape(n, H, -1) for x in "qkv")
    decay = key_decays(h, t["a1"], t["a2"], t["a2.b"], m["tau"]).reshape(n, H, -1)
    o, state = keyed_sums(q * m["dim"] ** -0.5, k, v, decay, state)
    return (head_norm(o, t["norm"], eps).reshape(n, -1) * silu(h @ t["g"].T)) @ t["o"].T, state


# ---- matrix memory with exponential gates -------------------------------------------------------------------------------------------
def memory_gates(h, t, cap):
    """(log input gate, log forget gate), [n, H] each."""
    soft = lambda z: cap * np.tanh(z / cap)  # noqa: E731
    return soft(h @ t["i"].T + t["i.b"]), log_sigmoid(soft(h @ t["f"].T + t["f.b"]))


def empty_memory(m):
    return np.zeros((m["heads"], m["dim"], m["vdim"])), np.zeros((m["heads"], m["dim"])), np.zeros(m["heads"])


def memory_reads(q, k, v, i, f, memory):
    """q, k [n, H, dim], v [n, H, vdim], i, f [n, H], memory (S [H, dim, vdim], sum of keys [H, dim], running maximum [H]).
    memory_reads.den: what each read was divided by."""
    s, z, m = memory
    out, dens = [], []
    for t in range(q.shape[0]):
        top = np.maximum(f[t] + m, i[t])
        keep, add = np.exp(f[t] + m - top), np.exp(i[t] - top)
        s = keep[:, None, None] * s + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        z = keep[:, None] * z + add[:, None] * k[t]
        m = top
        den = np.maximum(np.abs((z * q[t]).sum(-1)), np.exp(-m)) + 1e-6
        dens.append(den)
        out.append(np.einsum("hdv,hd->hv", s, q[t]) / den[:, None])
    memory_reads.den = np.asarray(dens)
    return np.asarray(out).reshape(q.shape[0], *v.shape[1:]), (s, z, m)


def matrix_memory(h, t, m, eps, memory):
    """(mixer output [n, width], new memory)."""
    n, H = h.shape[0], m["heads"]
    q, k, v = ((h @ t[x].T).reshape(n, H, -1) for x in "qkv")
    i, f = memory_gates(h, t, m["gate_cap"])
    o, memory = memory_reads(q * m["dim"] ** -0.5, k, v, i, f, memory)
    return (unit(o, eps).reshape(n, -1) * t["norm"] * sigmoid(h @ t["g"].T)) @ t["o"].T, memory


def side_by_side(left, right, m):
    return m["left_scale"] * left + m["right_scale"] * right


class PlainModel:
    """The whole decoder with the keys, values and states of every token seen so far; tensors: name -> float array."""

    def __init__(self, config, tensors):
        self.c, self.t = config, {k: np.asarray(v, np.float64) for k, v in tensors.items()}
        self.clear()

    def clear(self):
        self.kv, self.state = {}, {}
        self.n, self.streams = 0, []

    def owner(self, i):
        """The layer whose tensors layer i uses."""
        j = self.c["layers"][i].get("weights_of")
        return i if j is None else self.owner(j)

    def sub(self, prefix):
        return {k[len(prefix):]: v for k, v in self.t.items() if k.startswith(prefix)}

    def attention(self, i, h, pos, t, m, eps):
        q, k, v = queries_and_cells(h, pos, t, m, eps)
        old = self.kv.get(i)
        self.kv[i] = (k, v) if old is None else (np.concatenate([old[0], k]), np.concatenate([old[1], v]))
        k, v = self.kv[i]
        return window_attention(q, k, v, pos, np.arange(k.shape[0]), head_scale(t["temp"], m["scale"]), m["mask"]["size"]).reshape(h.shape[0], -1) @ t["o"].T

    def mix(self, i, h, pos):
        ly, eps, p = self.c["layers"][i], self.c["norm"]["eps"], f"l{self.owner(i)}.mix."
        m = ly["mixer"]
        if ly["type"] == "gla":
            y, self.state[i] = gla(h, self.sub(p), m, eps, self.state.get(i, np.zeros((m["heads"], m["dim"], m["vdim"]))))
            return y
        left = self.attention(i, h, pos, self.sub(p + "left."), m["left"], eps)
        right, self.state[i] = matrix_memory(h, self.sub(p + "right."), m["right"], eps, self.state.get(i, empty_memory(m["right"])))
        return side_by_side(left, right, m)

    def operand(self, x):
        """What the sublayers read of the residual stream."""
        return x

    def feed(self, tokens):
        """Logits [n, vocab] of the next tokens of the sequence; self.streams: the residual stream after every layer."""
        eps, alpha, t = self.c["norm"]["eps"], self.c["postln_alpha"], self.t
        tokens = [int(v) for v in tokens]
        pos = np.arange(self.n, self.n + len(tokens))
        self.n += len(tokens)
        x = embedding(tokens, t["embed"], self.c["embedding"]["scale"])
        self.streams = []
        for i, ly in enumerate(self.c["layers"]):
            p = f"l{self.owner(i)}."
            h = self.operand(x)
            x = norm_after_sum(x, gated(self.mix(i, h, pos), h, t[p + "rg1"], t[p + "rg1.b"]), alpha, t[p + "norm1"], eps)
            if ly["mlp"] is not None:
                h = self.operand(x)
                y = swiglu(h, t[p + "mlp.gate"], t[p + "mlp.up"], t[p + "mlp.down"])
                x = norm_after_sum(x, gated(y, h, t[p + "rg2"], t[p + "rg2.b"]), alpha, t[p + "norm2"], eps)
            self.streams.append(x)
        return rms_norm(x, t["final.norm"], eps) @ t["head"].T
