"""Pibalorn: a decoder of grouped-query attention and decayed linear-attention layers with one norm for both parts of a layer, clamped GLU
feed-forwards (dense, or experts beside a shared one), a bigram embedding, and a range of layers that runs several times with the same
weights.  This module reads its configuration into layer descriptions (pi_model_create_layers) and its tensors into the engine's roles; the
computation is the engine's."""
import numpy as np

from . import lib as pl
from .checkpoint import as_bf16, as_f32
from .model import LayerModel

GLU_GAIN = 1.702           # slope of the sigmoid in the GLU
SINK = 0.0                 # score of the soft-max's entry without a value


def layer_descs(config):
    out = []
    for i, layer in enumerate(config["layers"]):
        m, f = layer["mixer"], layer.get("mlp")
        d = dict(n_head=m["heads"], dim=m["dim"], vdim=m["vdim"], kv_from=-1, glu_gain=GLU_GAIN)
        if layer["type"] == "attention":
            rot = m.get("rot") or {"dims": 0, "base": 1.0}
            if m["vdim"] != m["dim"]:
                raise ValueError(f"layer {i}: the values are the keys, so vdim has to be dim")
            d.update(mixer=pl.MIXER_GROUPED, n_kv_head=m["kv_heads"], rot_dim=rot["dims"], rot_base=rot["base"], scale=m["scale"], values_are_keys=1, unit_qk=1, sink=SINK)
        elif layer["type"] == "lightning":
            if len(m["decay"]) != m["heads"]:
                raise ValueError(f"layer {i}: one decay per head")
            d.update(mixer=pl.MIXER_LINEAR)
        else:
            raise ValueError(f"layer {i}: mixer {layer['type']!r} is not part of this design")
        if f is None:
            d["ffn"] = pl.FFN_NONE
        elif f["kind"] == "dense":
            d.update(ffn=pl.FFN_GLU, glu_ff=f["ff"], glu_limit=f["limit"])
        elif f["kind"] == "moe":
            d.update(ffn=pl.FFN_GLU_MOE, n_expert=f["router"]["experts"], n_top=f["router"]["top"], expert_ff=f["expert"]["ff"], expert_limit=f["expert"]["limit"])
            if f.get("shared"):
                d.update(glu_ff=f["shared"]["ff"], glu_limit=f["shared"]["limit"])
        else:
            raise ValueError(f"layer {i}: feed-forward {f['kind']!r} is not part of this design")
        out.append(d)
    return out


def model_opts(config):
    e = config["embedding"]
    out = dict(embed_scale=e["scale"])
    b = e.get("bigram")
    if b:
        out.update(bigram_buckets=b["buckets"], bigram_mul_prev=b["mul_prev"], bigram_mul_cur=b["mul_cur"])
    loop = config.get("loop")
    if loop and loop["stop"] > loop["start"]:
        out.update(loop_start=loop["start"], loop_stop=loop["stop"], loop_times=loop["times"])
    return out


def build(config, tensors, compute=pl.BF16, n_ctx=4096, max_batch=0):
    """A finalized model from a configuration and its tensors (name -> bf16 bit patterns or floats, [out, in])."""
    descs, opts, t = layer_descs(config), model_opts(config), tensors
    m = LayerModel("pibalorn", descs, n_embd=config["width"], n_vocab=config["vocab"], n_ctx=n_ctx, norm_eps=config["norm"]["eps"], compute=compute, max_batch=max_batch, **opts)
    m.set_tensor(-1, "tok_embd", as_bf16(t["embed"]))
    m.set_tensor(-1, "output_norm", as_f32(t["final.norm"]))
    m.set_tensor(-1, "output", as_bf16(t["head"]))
    if "bigram_buckets" in opts:
        m.set_tensor(-1, "bigram", as_bf16(t["bigram"]))
    if "loop_times" in opts:
        m.set_tensor(-1, "loop_step", as_f32(t["loop.step"]))
    for i, d in enumerate(descs):
        p, q = f"l{i}.mix.", f"l{i}.mlp."
        m.set_tensor(i, "attn_norm", as_f32(t[f"l{i}.norm1"]))
        for role in ("q", "k") if d["mixer"] == pl.MIXER_GROUPED else ("q", "k", "v", "g"):
            m.set_tensor(i, "mix_" + role, as_bf16(t[p + role]))
        if d["mixer"] == pl.MIXER_LINEAR:
            m.set_tensor(i, "mix_norm", as_f32(t[p + "norm"]))
            m.set_tensor(i, "mix_decay", np.asarray(config["layers"][i]["mixer"]["decay"], np.float32))
        m.set_tensor(i, "wo", as_bf16(t[p + "o"]))
        if d.get("glu_ff"):
            one = q if d["ffn"] == pl.FFN_GLU else q + "shared."
            for role in ("gate", "up", "down"):
                m.set_tensor(i, "glu_" + role, as_bf16(t[one + role]))
        if d["ffn"] == pl.FFN_GLU_MOE:
            m.set_tensor(i, "router", as_bf16(t[q + "router"]))
            for role in ("gate", "up", "down"):
                m.set_tensor(i, "expert_" + role, np.concatenate([as_bf16(t[f"{q}e{e}.{role}"]) for e in range(d["n_expert"])]))
            if d.get("glu_ff"):
                m.set_tensor(i, "shared_score", as_bf16(t[q + "shared.sg"]))
    m.finalize()
    m.release_host()
    return m
