"""Small random Lerasun models for the tests: configurations, weights (bf16 values), and the error of logits against the oracle."""
import numpy as np

from powerinfer_amd.checkpoint import bf16_bits, bf16_floats


def layer(heads, dim, rot, vdim, rank, base=10000.0, scale=None, kv_from=None, moe=None):
    """moe: None, or (experts, top, group count, groups kept, ff)."""
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "rot": {"base": base, "dims": rot},
         "scale": (dim + rot) ** -0.5 if scale is None else scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    f = None
    if moe is not None:
        e, top, g, keep, ff = moe
        f = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": e, "top": top, "groups": {"count": g, "keep": keep}}}
    return {"type": "latent_attention", "mixer": m, "mlp": f}


def config(width, vocab, layers, logit_scale=0.7, eps=1e-5):
    return {"architecture": "Lerasun", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps}, "logit_scale": logit_scale}


# every layer different: head counts and sizes that are no multiples of anything, two rotations, shared cells twice, a layer without
# experts, groups of one expert, one single group
def odd_config():
    return config(100, 131, [
        layer(3, 24, 16, 40, 50, moe=(6, 2, 3, 2, 24)),
        layer(5, 17, 16, 9, 50, kv_from=0, scale=0.3),
        layer(2, 40, 6, 16, 72, base=500.0, moe=(9, 3, 1, 1, 33)),
        layer(1, 8, 6, 130, 72, base=500.0, kv_from=2, moe=(4, 1, 4, 3, 8)),
        layer(7, 16, 16, 24, 50, kv_from=0, moe=(8, 8, 2, 2, 16)),
    ], logit_scale=1.3)


# sizes every fast path takes: long prompt runs expand keys and values, steps of few tokens run fused
def even_config():
    return config(192, 200, [
        layer(4, 32, 16, 32, 64, moe=(16, 3, 4, 2, 48)),
        layer(6, 32, 16, 64, 64, kv_from=0, moe=(12, 2, 6, 4, 64)),
        layer(3, 64, 32, 64, 160, base=50000.0),
    ], logit_scale=0.5)


def weights(cfg, seed):
    """name -> float32 arrays holding bf16 values."""
    rng = np.random.default_rng(seed)
    t = {}

    def mat(name, rows, cols, gain=1.0):
        t[name] = rng.standard_normal((rows, cols)).astype(np.float32) * np.float32(gain / np.sqrt(cols))

    def vec(name, n, mean, std):
        t[name] = (mean + std * rng.standard_normal(n)).astype(np.float32)

    d, v = cfg["width"], cfg["vocab"]
    t["embed"] = rng.standard_normal((v, d)).astype(np.float32)
    vec("embed.norm", d, 0.0, 0.2)
    vec("final.norm", d, 0.0, 0.2)
    mat("head", v, d, 2.0)
    for i, ly in enumerate(cfg["layers"]):
        m, p = ly["mixer"], f"l{i}.mix."
        vec(f"l{i}.norm1", d, 0.0, 0.2)
        mat(p + "q", m["heads"] * (m["dim"] + m["rot_dim"]), d, 1.5)
        if "kv_from" not in m:
            mat(p + "dkv", m["kv_rank"] + m["rot_dim"], d)
            vec(p + "dkv.norm", m["kv_rank"], 1.0, 0.2)
        mat(p + "uk", m["heads"] * m["dim"], m["kv_rank"], 1.5)
        mat(p + "uv", m["heads"] * m["vdim"], m["kv_rank"])
        vec(p + "sink", m["heads"], 1.0, 1.5)
        mat(p + "o", d, m["heads"] * m["vdim"])
        if ly["mlp"] is None:
            continue
        p, f = f"l{i}.mlp.", ly["mlp"]
        vec(f"l{i}.norm2", d, 0.0, 0.2)
        e = f["router"]["experts"]
        mat(p + "router", e, d, 1.5)
        vec(p + "correction", e, -0.2, 0.4)
        for k in range(e):
            mat(f"{p}e{k}.up", f["expert"]["ff"], d)
            mat(f"{p}e{k}.down", d, f["expert"]["ff"])
    return {k: bf16_floats(bf16_bits(a)).reshape(a.shape) for k, a in t.items()}


def tokens(cfg, n, seed):
    return [int(v) for v in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


def row_errors(got, want):
    """Root mean square over the vocabulary of the difference (mean taken off), relative to the spread of the expected logits."""
    d = np.asarray(got, np.float64) - want
    d -= d.mean(axis=1, keepdims=True)
    return np.sqrt((d ** 2).mean(axis=1)) / np.asarray(want).std()
