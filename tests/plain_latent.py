"""Plain, slow implementations (numpy, float64) of the mechanisms of the layer-described decoder models, one function per mechanism:
the oracle of tests/test_*lerasun*.py and tests/test_gpu_latent_ops.py.  Nothing here is shared with powerinfer_amd/.

Weights are float arrays [out, in]; x rows are tokens.
"""
import numpy as np


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm_zero(x, w, eps):
    """RMS norm whose stored weight is the distance from one."""
    return rms(x, eps) * (1.0 + w)


def rms_norm_plain(x, w, eps):
    return rms(x, eps) * w


def rotate_pairs(x, pos, base):
    """Rotary embedding, neighbours (2i, 2i+1) forming pair i; x [..., n_tok, dims], pos [n_tok]."""
    dims = x.shape[-1]
    f = float(base) ** (-2.0 * np.arange(dims // 2) / dims)
    a = np.asarray(pos, np.float64)[:, None] * f[None, :]
    c, s = np.cos(a), np.sin(a)
    u, v = x[..., 0::2], x[..., 1::2]
    out = np.empty_like(x)
    out[..., 0::2] = u * c - v * s
    out[..., 1::2] = v * c + u * s
    return out


def latent_of(h, w_dkv, norm_w, kv_rank, pos, base, eps):
    """(latent [n, kv_rank], rotated shared key part [n, rot_dim]) of the tokens h."""
    z = h @ w_dkv.T
    return rms_norm_plain(z[:, :kv_rank], norm_w, eps), rotate_pairs(z[:, kv_rank:], pos, base)


def sink_softmax(scores, sink):
    """Soft-max over the last axis whose denominator also holds exp(sink); scores may contain -inf."""
    m = np.maximum(scores.max(axis=-1), sink)
    e = np.exp(scores - m[..., None])
    return e / (e.sum(axis=-1) + np.exp(sink - m))[..., None]


def latent_attention(h, pos, c, k_rot, kpos, t, cfg):
    """Queries from h at positions pos against the latents c and rotated key parts k_rot at positions kpos.
    t: q [H (dim + rot), d], uk [H dim, rank], uv [H vdim, rank], sink [H], o [d, H vdim]."""
    H, D, R, V = cfg["heads"], cfg["dim"], cfg["rot_dim"], cfg["vdim"]
    n, m = h.shape[0], c.shape[0]
    q = (h @ t["q"].T).reshape(n, H, D + R)
    k = (c @ t["uk"].T).reshape(m, H, D)
    v = (c @ t["uv"].T).reshape(m, H, V)
    visible = np.asarray(kpos)[None, :] <= np.asarray(pos)[:, None]
    out = np.empty((n, H, V))
    for a in range(H):
        q_rot = rotate_pairs(q[:, a, D:], pos, cfg["rot"]["base"])
        s = (q[:, a, :D] @ k[:, a].T + q_rot @ k_rot.T) * cfg["scale"]
        s = np.where(visible, s, -np.inf)
        out[:, a] = sink_softmax(s, np.full(n, t["sink"][a])) @ v[:, a]
    return out.reshape(n, H * V) @ t["o"].T


def route(h, w_router, correction, top, groups, keep):
    """(chosen expert ids [n, top] by falling choice score, their weights).  route.margins: per token, how far the closest decision was."""
    s = 1.0 / (1.0 + np.exp(-(h @ w_router.T)))
    ids, wts, margins = [], [], []
    for row in s:
        choice = row + correction
        size = choice.size // groups
        best = [np.sort(choice[g * size:(g + 1) * size])[::-1][:2].sum() for g in range(groups)]
        kept = np.argsort(-np.asarray(best), kind="stable")[:keep]
        open_ = np.full(choice.size, -np.inf)
        for g in kept:
            open_[g * size:(g + 1) * size] = choice[g * size:(g + 1) * size]
        order = np.argsort(-open_, kind="stable")
        e = order[:top]
        gaps = [open_[order[top - 1]] - open_[order[top]]] if top < choice.size else [np.inf]
        if keep < groups:
            by = np.sort(best)[::-1]
            gaps.append(by[keep - 1] - by[keep])
        margins.append(min(gaps))
        ids.append(e)
        wts.append(row[e] / (row[e].sum() + 1e-20))
    route.margins = np.asarray(margins)
    return np.asarray(ids), np.asarray(wts)


def expert(h, up, down):
    return np.square(np.maximum(h @ up.T, 0.0)) @ down.T


def mixture(h, t, cfg):
    r = cfg["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    ids, w = route(h, t["router"], t["correction"], r["top"], g["count"], g["keep"])
    out = np.zeros((h.shape[0], t["down"][0].shape[0]))
    for i in range(h.shape[0]):
        for e, we in zip(ids[i], w[i]):
            out[i] += we * expert(h[i:i + 1], t["up"][e], t["down"][e])[0]
    return out


class PlainModel:
    """The whole decoder, holding the latents of every token seen so far; tensors: name -> float array."""

    def __init__(self, config, tensors):
        self.c, self.t = config, {k: np.asarray(v, np.float64) for k, v in tensors.items()}
        self.clear()

    def clear(self):
        self.kv = {}
        self.n = 0
        self.streams = []
        self.margins = np.empty(0)                   # closest routing decision of every token so far

    def _mix(self, i, h, pos):
        m, p = self.c["layers"][i]["mixer"], f"l{i}.mix."
        src = m.get("kv_from")
        if src is None:
            lat, kr = latent_of(h, self.t[p + "dkv"], self.t[p + "dkv.norm"], m["kv_rank"], pos, m["rot"]["base"], self.c["norm"]["eps"])
            old = self.kv.get(i)
            self.kv[i] = (lat, kr) if old is None else (np.vstack([old[0], lat]), np.vstack([old[1], kr]))
            src = i
        lat, kr = self.kv[src]
        return latent_attention(h, pos, lat, kr, np.arange(lat.shape[0]), {k: self.t[p + k] for k in ("q", "uk", "uv", "sink", "o")}, m)

    def _ff(self, i, h):
        f = self.c["layers"][i]["mlp"]
        if f is None:
            return 0.0
        p = f"l{i}.mlp."
        E = f["router"]["experts"]
        return mixture(h, {"router": self.t[p + "router"], "correction": self.t[p + "correction"],
                           "up": [self.t[f"{p}e{e}.up"] for e in range(E)], "down": [self.t[f"{p}e{e}.down"] for e in range(E)]}, f)

    def feed(self, tokens):
        """Logits [n, vocab] of the next tokens of the sequence; self.streams: the residual stream after every layer."""
        eps = self.c["norm"]["eps"]
        pos = np.arange(self.n, self.n + len(tokens))
        self.n += len(tokens)
        x = rms_norm_zero(self.t["embed"][np.asarray(tokens)], self.t["embed.norm"], eps)
        self.streams = []
        margins = np.full(len(tokens), np.inf)
        for i in range(len(self.c["layers"])):
            a = rms_norm_zero(x, self.t[f"l{i}.norm1"], eps)
            y = self._mix(i, a, pos)
            if self.c["layers"][i]["mlp"] is not None:
                y = y + self._ff(i, rms_norm_zero(x, self.t[f"l{i}.norm2"], eps))
                margins = np.minimum(margins, getattr(route, "margins", margins))
            x = x + y
            self.streams.append(x)
        self.margins = np.concatenate([self.margins, margins])
        return rms_norm_zero(x, self.t["final.norm"], eps) @ self.t["head"].T * self.c["logit_scale"]
