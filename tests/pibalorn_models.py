"""Small random Pibalorn models for the tests: configurations and weights (bf16 values)."""
import numpy as np

from powerinfer_amd.checkpoint import bf16_bits, bf16_floats


def dense(ff, limit=1.4):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, top, ff, limit=1.8, shared=None):
    """shared: None, or (ff, limit)."""
    out = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit}}
    if shared:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


def attention(heads, kv_heads, dim, rot=None, base=10000.0, scale=None, mlp=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "rot": {"dims": dim if rot is None else rot, "base": base},
                                           "scale": dim ** -0.5 if scale is None else scale}, "mlp": mlp}


def lightning(heads, dim, vdim, decay, mlp=None):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}, "mlp": mlp}


def config(width, vocab, layers, loop=None, eps=1e-5, scale=3.0, bigram=(97, 29, 13)):
    """loop: None, or (start, stop, times); bigram: (buckets, mul_prev, mul_cur)."""
    c = {"architecture": "Pibalorn", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps},
         "embedding": {"scale": scale, "bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


# every layer different: sizes that are no multiples of anything, a part of the head rotated, values wider and narrower than keys, no
# feed-forward, one and many key heads, decays from nothing to everything, a loop of one layer that starts the model
def odd_config():
    return config(100, 131, [
        lightning(3, 20, 36, (1.0, 0.5, 0.03), mlp=moe(7, 3, 23, 0.7)),
        attention(6, 2, 40, rot=24, base=500.0, mlp=dense(90, 0.9)),
        attention(5, 1, 17, rot=6, scale=0.4),
        lightning(5, 33, 9, (0.999, 0.9, 0.0, 0.7, 0.97), mlp=dense(33, 3.0)),
        attention(4, 4, 130, rot=2, mlp=moe(20, 18, 9, 1.1, (31, 0.8))),
    ], loop=(0, 1, 3), scale=2.5, bigram=(41, 5, 1000003))


# sizes like those of larger models, two layers of different kinds in the loop
def even_config():
    return config(192, 200, [
        attention(8, 2, 64, mlp=dense(256)),
        lightning(4, 64, 64, (0.999, 0.98, 0.9, 0.5), mlp=moe(18, 5, 48, shared=(64, 1.2))),
        attention(6, 3, 32, base=50000.0, mlp=moe(12, 2, 64, 1.3, (32, 1.7))),
        lightning(2, 128, 128, (0.995, 0.6), mlp=moe(8, 1, 32)),
    ], loop=(1, 3, 2))


# the remaining head sizes of the kernels, the loop over the whole model
def tall_config():
    return config(136, 90, [
        attention(4, 2, 96, mlp=dense(64)),
        lightning(2, 160, 200, (0.99, 0.8), mlp=dense(48)),
        attention(3, 1, 192, rot=64),
        attention(2, 2, 256, rot=128, mlp=moe(4, 2, 16, shared=(8, 1.0))),
        lightning(3, 96, 70, (0.9, 1.0, 0.2)),
    ], loop=(0, 5, 2), bigram=(1, 3, 2))


def weights(cfg, seed):
    """name -> float32 arrays holding bf16 values."""
    rng = np.random.default_rng(seed)
    t = {}

    def mat(name, rows, cols, gain=1.0):
        t[name] = rng.standard_normal((rows, cols)).astype(np.float32) * np.float32(gain / np.sqrt(cols))

    def vec(name, n, mean, std):
        t[name] = (mean + std * rng.standard_normal(n)).astype(np.float32)

    d, v = cfg["width"], cfg["vocab"]
    t["embed"] = (rng.standard_normal((v, d)) / cfg["embedding"]["scale"]).astype(np.float32)
    t["bigram"] = (0.5 * rng.standard_normal((cfg["embedding"]["bigram"]["buckets"] + 1, d))).astype(np.float32)
    if "loop" in cfg:
        t["loop.step"] = (0.5 * rng.standard_normal((cfg["loop"]["times"], d))).astype(np.float32)
    vec("final.norm", d, 1.0, 0.2)
    mat("head", v, d, 2.0)
    for i, ly in enumerate(cfg["layers"]):
        m, p, f = ly["mixer"], f"l{i}.mix.", ly["mlp"]
        H = m["heads"]
        vec(f"l{i}.norm1", d, 1.0, 0.2)
        if ly["type"] == "attention":
            mat(p + "q", H * m["dim"], d)
            mat(p + "k", m["kv_heads"] * m["dim"], d)
        else:
            mat(p + "q", H * m["dim"], d)
            mat(p + "k", H * m["dim"], d)
            mat(p + "v", H * m["vdim"], d)
            mat(p + "g", H * m["vdim"], d)
            vec(p + "norm", H * m["vdim"], 1.0, 0.2)
        mat(p + "o", d, H * m["vdim"])

        def glu(q, ff):
            mat(q + "gate", ff, d, 1.5)
            mat(q + "up", ff, d, 1.5)
            mat(q + "down", d, ff)

        q = f"l{i}.mlp."
        if f and f["kind"] == "dense":
            glu(q, f["ff"])
        elif f:
            mat(q + "router", f["router"]["experts"], d, 1.5)
            for e in range(f["router"]["experts"]):
                glu(f"{q}e{e}.", f["expert"]["ff"])
            if "shared" in f:
                glu(q + "shared.", f["shared"]["ff"])
                mat(q + "shared.sg", 1, d)
    return {k: bf16_floats(bf16_bits(a)).reshape(a.shape) for k, a in t.items()}
