"""Small random Fikevik models for the tests: configurations and weights (bf16 values)."""
import numpy as np

from powerinfer_amd.checkpoint import bf16_bits, bf16_floats


def dense(ff):
    return {"kind": "dense", "ff": ff}


def gla(heads, dim, vdim, tau=16.0, mlp=None, of=None):
    """of: the layer whose weights it uses."""
    return shared({"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "mlp": mlp}, of)


def parallel(left, right, left_scale=0.7, right_scale=0.8, mlp=None, of=None):
    """left: attention(...), right: memory(...)."""
    return shared({"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}, "mlp": mlp}, of)


def attention(heads, kv_heads, dim, vdim, window, rot=None, base=10000.0, scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window}, "rot": {"dims": dim // 2 * 2 if rot is None else rot, "base": base},
            "scale": dim ** -0.5 if scale is None else scale}


def memory(heads, dim, vdim, cap=15.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def shared(layer, of):
    return layer if of is None else dict(layer, weights_of=of)


def config(width, vocab, layers, eps=1e-5, scale=1.5, alpha=1.7):
    return {"architecture": "Fikevik", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps}, "embedding": {"scale": scale}, "postln_alpha": alpha}


# every layer different: sizes that are no multiples of anything, a part of the head rotated, values wider and narrower than keys, no feed-forward,
# strong decays, a window of one position, a single head
def odd_config():
    return config(100, 131, [
        parallel(attention(6, 2, 40, 24, 21, rot=24, base=500.0), memory(3, 20, 36, cap=4.0), 0.4, 1.1, mlp=dense(90)),
        gla(3, 33, 9, tau=0.7, mlp=dense(33)),
        gla(1, 17, 70, tau=5.0),
        parallel(attention(5, 1, 17, 50, 1, rot=6, scale=0.4), memory(1, 9, 13), 1.3, 0.5),
        gla(5, 20, 36, tau=2.0, mlp=dense(7)),
    ], scale=2.5, alpha=1.0)


# sizes like those of larger models, layers that share weights in either order
def even_config():
    a, b = parallel(attention(8, 2, 64, 64, 48, base=50000.0), memory(4, 64, 64), mlp=dense(256)), gla(4, 64, 64, mlp=dense(320))
    return config(192, 200, [b, a, shared(b, 0), shared(a, 4), dict(a), gla(2, 128, 128, tau=8.0, mlp=dense(128)), shared(a, 4)], alpha=2.3)


# the remaining head sizes of the kernels
def tall_config():
    return config(136, 90, [
        parallel(attention(4, 2, 96, 130, 100), memory(2, 160, 200, cap=8.0), mlp=dense(64)),
        gla(2, 160, 200, tau=4.0, mlp=dense(48)),
        parallel(attention(2, 2, 256, 192, 400, rot=128), memory(3, 96, 70, cap=20.0), 0.9, 0.2),
        gla(2, 256, 256, tau=16.0),
        gla(3, 96, 70, tau=1.0, mlp=dense(200)),
    ], alpha=1.4)


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
    vec("final.norm", d, 1.0, 0.2)
    mat("head", v, d, 2.0)
    for i, ly in enumerate(cfg["layers"]):
        if "weights_of" in ly:
            continue
        m, p, f = ly["mixer"], f"l{i}.mix.", ly["mlp"]
        for part in "12" if f else "1":
            vec(f"l{i}.norm{part}", d, 1.0, 0.2)
            mat(f"l{i}.rg{part}", d, d)
            vec(f"l{i}.rg{part}.b", d, 0.5, 0.5)
        if ly["type"] == "gla":
            H, rank = m["heads"], 5 + 3 * i
            for x, n in (("q", H * m["dim"]), ("k", H * m["dim"]), ("v", H * m["vdim"]), ("g", H * m["vdim"]), ("a1", rank)):
                mat(p + x, n, d)
            mat(p + "a2", H * m["dim"], rank, 2.0)
            vec(p + "a2.b", H * m["dim"], 0.0, 3.0)
            vec(p + "norm", m["vdim"], 1.0, 0.2)
            mat(p + "o", d, H * m["vdim"])
        else:
            a, r = m["left"], m["right"]
            H, G = a["heads"], a["kv_heads"]
            for x, n in (("q", H * a["dim"]), ("k", G * a["dim"]), ("v", G * a["vdim"])):
                mat(p + "left." + x, n, d)
            for x in ("q.norm", "k.norm"):
                vec(p + "left." + x, a["dim"], 1.3, 0.3)
            vec(p + "left.temp", H, 1.0, 0.4)
            mat(p + "left.o", d, H * a["vdim"])
            M = r["heads"]
            for x, n in (("q", M * r["dim"]), ("k", M * r["dim"]), ("v", M * r["vdim"]), ("g", M * r["vdim"]), ("i", M), ("f", M)):
                mat(p + "right." + x, n, d)
            vec(p + "right.i.b", M, 0.0, 2.0)
            vec(p + "right.f.b", M, 3.0, 2.0)
            vec(p + "right.norm", M * r["vdim"], 1.0, 0.2)
            mat(p + "right.o", d, M * r["vdim"])
        if f:
            for x, rows, cols in (("gate", f["ff"], d), ("up", f["ff"], d), ("down", d, f["ff"])):
                mat(f"l{i}.mlp.{x}", rows, cols, 1.5)
    return {k: bf16_floats(bf16_bits(a)).reshape(a.shape) for k, a in t.items()}
