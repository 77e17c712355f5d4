"""Lerasun: a decoder of latent-attention layers with soft-max sinks and grouped sigmoid routing over small experts, attention and
experts side by side.  This module reads its configuration into layer descriptions (pi_model_create_layers) and its tensors into the
engine's roles; the computation is the engine's."""
import numpy as np

from . import lib as pl
from .checkpoint import as_bf16, as_f32
from .model import LayerModel

NORM_OFFSET = 1.0          # the model's own norms store their weights around zero


def layer_descs(config):
    out = []
    for i, layer in enumerate(config["layers"]):
        if layer["type"] != "latent_attention":
            raise ValueError(f"layer {i}: mixer {layer['type']!r} is not part of this design")
        m, f = layer["mixer"], layer.get("mlp")
        src = m.get("kv_from")
        d = dict(mixer=pl.MIXER_LATENT, n_head=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"], vdim=m["vdim"], kv_rank=m["kv_rank"],
                 kv_from=-1 if src is None else src, scale=m["scale"], rot_base=m["rot"]["base"])
        if m["rot"].get("dims", m["rot_dim"]) != m["rot_dim"]:
            raise ValueError(f"layer {i}: the rotation covers the whole rotated part")
        if f is None:
            d["ffn"] = pl.FFN_NONE
        elif f["kind"] == "moe":
            r = f["router"]
            g = r.get("groups") or {"count": 1, "keep": 1}
            d.update(ffn=pl.FFN_MOE, n_expert=r["experts"], n_top=r["top"], n_group=g["count"], n_group_keep=g["keep"], expert_ff=f["expert"]["ff"])
        else:
            raise ValueError(f"layer {i}: feed-forward {f['kind']!r} is not part of this design")
        out.append(d)
    return out


def build(config, tensors, compute=pl.BF16, n_ctx=4096, max_batch=0):
    """A finalized model from a configuration and its tensors (name -> bf16 bit patterns or floats, [out, in])."""
    descs = layer_descs(config)
    m = LayerModel("lerasun", descs, n_embd=config["width"], n_vocab=config["vocab"], n_ctx=n_ctx, norm_eps=config["norm"]["eps"], compute=compute,
                   logit_scale=config["logit_scale"], norm_offset=NORM_OFFSET, max_batch=max_batch)
    t = tensors
    m.set_tensor(-1, "tok_embd", as_bf16(t["embed"]))
    m.set_tensor(-1, "embd_norm", as_f32(t["embed.norm"]))
    m.set_tensor(-1, "output_norm", as_f32(t["final.norm"]))
    m.set_tensor(-1, "output", as_bf16(t["head"]))
    for i, d in enumerate(descs):
        p = f"l{i}.mix."
        m.set_tensor(i, "attn_norm", as_f32(t[f"l{i}.norm1"]))
        m.set_tensor(i, "mix_q", as_bf16(t[p + "q"]))
        if d["kv_from"] < 0:
            m.set_tensor(i, "mix_dkv", as_bf16(t[p + "dkv"]))
            m.set_tensor(i, "mix_dkv_norm", as_f32(t[p + "dkv.norm"]))
        m.set_tensor(i, "mix_uk", as_bf16(t[p + "uk"]))
        m.set_tensor(i, "mix_uv", as_bf16(t[p + "uv"]))
        m.set_tensor(i, "mix_sink", as_f32(t[p + "sink"]))
        m.set_tensor(i, "wo", as_bf16(t[p + "o"]))
        if d["ffn"] == pl.FFN_NONE:
            continue
        p = f"l{i}.mlp."
        m.set_tensor(i, "ffn_norm", as_f32(t[f"l{i}.norm2"]))
        m.set_tensor(i, "router", as_bf16(t[p + "router"]))
        m.set_tensor(i, "router_bias", as_f32(t[p + "correction"]))
        m.set_tensor(i, "expert_up", np.concatenate([as_bf16(t[f"{p}e{e}.up"]) for e in range(d["n_expert"])]))
        m.set_tensor(i, "expert_down", np.concatenate([as_bf16(t[f"{p}e{e}.down"]) for e in range(d["n_expert"])]))
    m.finalize()
    m.release_host()
    return m
