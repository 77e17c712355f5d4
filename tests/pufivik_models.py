"""Small random Pufivik models for the tests: configurations and weights (bf16 values)."""
import numpy as np

from powerinfer_amd.checkpoint import bf16_bits, bf16_floats


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def mixer(heads, kv_heads, dim, vdim, scale, v_mix, rot):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale, "v_mix": v_mix, "rot": rot}


def talking(heads, kv_heads, dim, vdim, mlp=None, rot=None, base=10000.0, factor=8.0, low=1.0, high=4.0, original=64, scale=None, v_mix=True):
    """Attention with sinks, mixed and gated heads."""
    r = {"base": base, "dims": dim // 2 * 2 if rot is None else rot, "scaling": {"factor": factor, "low": low, "high": high, "original": original}}
    return {"type": "attention", "mixer": mixer(heads, kv_heads, dim, vdim, scale, v_mix, r), "mlp": mlp}


def capped(heads, kv_heads, dim, vdim, cap, mlp=None, rot=None, base=10000.0, factor=4.0, slow=1.0, fast=32.0, original=64, scale=None, v_mix=True):
    """Attention with soft-capped scores."""
    r = {"base": base, "dims": dim // 2 * 2 if rot is None else rot, "scaling": {"factor": factor, "fast": fast, "slow": slow, "original": original}}
    return {"type": "attention_2", "mixer": dict(mixer(heads, kv_heads, dim, vdim, scale, v_mix, r), softcap=cap), "mlp": mlp}


def config(width, vocab, layers, groups=1, taps=4, eps=1e-5, scale=1.5, mult=0.8):
    return {"architecture": "Pufivik", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps, "groups": groups}, "embedding": {"scale": scale}, "residual_mult": mult,
            "canon": {"taps": taps}}


# every layer different: sizes that are no multiples of anything, a part of the head rotated, values wider and narrower than keys, no feed-forward,
# one head, a single expert, layers that leave the values alone (the first among them), three taps fewer than the width has groups
def odd_config():
    return config(100, 131, [
        capped(5, 1, 17, 50, 5.0, rot=6, scale=0.4, original=20, v_mix=False),
        talking(6, 2, 40, 24, mlp=moe(5, 2, 30), rot=24, base=500.0, original=40),
        capped(4, 2, 33, 24, 2.0, mlp=moe(1, 1, 17), rot=32, base=300.0, factor=2.5, slow=0.5, fast=6.0, original=100),
        talking(1, 1, 20, 70, rot=4, factor=3.0, low=0.5, high=9.0, v_mix=False),
        talking(2, 2, 24, 24, mlp=moe(9, 3, 33), rot=20),
        capped(8, 2, 24, 24, 11.0, mlp=moe(3, 3, 50), rot=10),
    ], groups=5, taps=3, scale=2.5, mult=1.0)


# sizes like those of larger models
def even_config():
    f = moe(12, 4, 64)
    t, c = talking(16, 4, 64, 64, f, base=50000.0, original=128), capped(16, 4, 64, 64, 25.0, f, original=256)
    return config(256, 200, [t, c, c, t, dict(c, mlp=None)], groups=8, taps=4, mult=0.6)


# the remaining head sizes of the kernels, one group of keys for many heads and one for each, a long convolution
def tall_config():
    return config(136, 90, [
        capped(4, 2, 96, 130, 20.0, moe(6, 1, 48)),
        talking(2, 2, 256, 192, rot=128, v_mix=False),
        talking(20, 1, 48, 72, moe(12, 2, 24), v_mix=False),
        capped(2, 1, 160, 200, 8.0, v_mix=False),
        talking(4, 1, 128, 100, moe(4, 2, 40), v_mix=False),
    ], groups=2, taps=7, mult=1.3)


def weights(cfg, seed, decided=False):
    """name -> float32 arrays holding bf16 values.  decided: the routers look at the first values of the embedding alone, which differ clearly and which no
    sublayer writes to, so that no choice of experts is a close call that rounding turns."""
    rng = np.random.default_rng(seed)
    t = {}

    def mat(name, rows, cols, gain=1.0):
        t[name] = rng.standard_normal((rows, cols)).astype(np.float32) * np.float32(gain / np.sqrt(cols))

    def vec(name, n, mean, std):
        t[name] = (mean + std * rng.standard_normal(n)).astype(np.float32)

    d, v = cfg["width"], cfg["vocab"]
    t["embed"] = (rng.standard_normal((v, d)) / cfg["embedding"]["scale"]).astype(np.float32)
    vec("final.norm", d, 1.0, 0.2)
    for i, ly in enumerate(cfg["layers"]):
        m, p, f = ly["mixer"], f"l{i}.mix.", ly["mlp"]
        H, G = m["heads"], m["kv_heads"]
        for x in ("norm1", "norm1b") + (("norm2", "norm2b") if f else ()):
            vec(f"l{i}.{x}", d, 1.0, 0.2)
        t[f"l{i}.canon1"] = (0.4 * rng.standard_normal((d, cfg["canon"]["taps"]))).astype(np.float32)
        for x, n in (("q", H * m["dim"]), ("k", G * m["dim"]), ("v", G * m["vdim"])):
            mat(p + x, n, d, 1.2)
        t[p + "vmix"] = np.float32(0.2 + 0.5 * rng.random())
        if ly["type"] == "attention":
            t[p + "talk"] = (np.eye(H) + 0.4 * rng.standard_normal((H, H))).astype(np.float32)
            vec(p + "sink", H, 0.5, 1.5)
            mat(p + "g", H, d, 1.5)
        mat(p + "o", d, H * m["vdim"])
        if f:
            mat(f"l{i}.mlp.router", f["router"]["experts"], d, 1.5)
            for e in range(f["router"]["experts"]):
                for x, rows, cols in (("gate", f["expert"]["ff"], d), ("up", f["expert"]["ff"], d), ("down", d, f["expert"]["ff"])):
                    mat(f"l{i}.mlp.e{e}.{x}", rows, cols, 1.5)
    if decided:
        n = max([ly["mlp"]["router"]["experts"] for ly in cfg["layers"] if ly["mlp"]] + [1])
        assert n <= d // cfg["norm"]["groups"]
        t["embed"][:, :n] = [2.5 * rng.permutation(np.linspace(-1, 1, n)) for _ in range(v)]
        t["embed"][:, :n] /= cfg["embedding"]["scale"]
        for i, ly in enumerate(cfg["layers"]):
            if ly["mlp"]:
                e = ly["mlp"]["router"]["experts"]
                t[f"l{i}.norm1b"][:n] = t[f"l{i}.norm2b"][:n] = 0
                t[f"l{i}.norm2"][:n] = 1
                t[f"l{i}.mlp.router"][:] = 0
                t[f"l{i}.mlp.router"][rng.permutation(e), np.arange(e)] = 1.5
            else:
                t[f"l{i}.norm1b"][:n] = 0
    return {k: bf16_floats(bf16_bits(a)).reshape(np.shape(a)) for k, a in t.items()}
