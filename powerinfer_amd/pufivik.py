"""Pufivik: a decoder with a norm (in groups) before and after every sublayer, a short convolution over time on what every mixer reads, grouped-query
attention of two kinds - with a sink per head, soft-max weights mixed over the heads and gated heads, or with soft-capped scores -, values mixed
with those of the first layer, and small experts chosen by sigmoid scores that multiply their input.  This module reads its configuration into layer
descriptions (pi_model_create_layers) and its tensors into the engine's roles; the computation is the engine's."""
import numpy as np

from . import lib as pl
from .checkpoint import as_bf16, as_f32
from .model import LayerModel

NO_LIMIT = float("inf")    # the experts' GLU is not clamped
SILU_GAIN = 1.0


def rotation(rot, pairs, kind, low, high):
    """low, high: the names of the scaling's constants for few and for many turns."""
    if not rot:
        return dict(rot_dim=0, rot_base=1.0)
    out, s = dict(rot_dim=rot["dims"], rot_base=rot["base"], rot_pairs=pairs), rot.get("scaling")
    if s:
        out.update(rot_scaling=kind, rot_factor=s["factor"], rot_original=s["original"], rot_low=s[low], rot_high=s[high])
    return out


def layer_descs(config):
    out = []
    for i, layer in enumerate(config["layers"]):
        m, f = layer["mixer"], layer.get("mlp")
        d = dict(mixer=pl.MIXER_GROUPED, kv_from=-1, n_head=m["heads"], n_kv_head=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], scale=m["scale"], sink=-NO_LIMIT,
                 value_mix=int(bool(m.get("v_mix"))))
        if layer["type"] == "attention":
            d.update(rotation(m.get("rot"), 0, pl.ROT_WAVES, "low", "high"), head_sinks=1, head_mix=1, head_gate=1)
        elif layer["type"] == "attention_2":
            d.update(rotation(m.get("rot"), 1, pl.ROT_RAMP, "slow", "fast"), softcap=m["softcap"])
        else:
            raise ValueError(f"layer {i}: mixer {layer['type']!r} is not part of this design")
        if f is None:
            d["ffn"] = pl.FFN_NONE
        elif f["kind"] == "moe":
            d.update(ffn=pl.FFN_GLU_MOE, n_expert=f["router"]["experts"], n_top=f["router"]["top"], expert_ff=f["expert"]["ff"], expert_limit=NO_LIMIT, glu_limit=NO_LIMIT, glu_gain=SILU_GAIN,
                     glu_plain_up=1, route_scores=1, weigh_input=1)
        else:
            raise ValueError(f"layer {i}: feed-forward {f['kind']!r} is not part of this design")
        out.append(d)
    return out


def model_opts(config):
    return dict(embed_scale=config["embedding"]["scale"], both_norms=1, residual_mult=config["residual_mult"], norm_groups=config["norm"]["groups"], conv_taps=config["canon"]["taps"])


def layer_tensors(d, t, i, keeps_values):
    """(role, array) of a layer; keeps_values: it is the first that mixes values, and its own go into the others'."""
    p, x, bf, f32 = f"l{i}.", f"l{i}.mix.", as_bf16, as_f32
    yield "attn_norm", f32(t[p + "norm1"])
    yield "attn_norm_after", f32(t[p + "norm1b"])
    yield "mix_conv", np.ascontiguousarray(f32(t[p + "canon1"]).T)
    for role in ("q", "k", "v"):
        yield "mix_" + role, bf(t[x + role])
    if d.get("head_mix"):
        yield "mix_sink", f32(t[x + "sink"])
        yield "mix_talk", f32(t[x + "talk"])
        yield "mix_head_gate", bf(t[x + "g"])
    if d["value_mix"] and not keeps_values:
        yield "mix_value", np.reshape(f32(t[x + "vmix"]), 1)
    yield "wo", bf(t[x + "o"])
    if d["ffn"] == pl.FFN_GLU_MOE:
        yield "ffn_norm", f32(t[p + "norm2"])
        yield "ffn_norm_after", f32(t[p + "norm2b"])
        yield "router", bf(t[p + "mlp.router"])
        for role in ("gate", "up", "down"):
            yield "expert_" + role, np.concatenate([bf(t[f"{p}mlp.e{e}.{role}"]) for e in range(d["n_expert"])])


def build(config, tensors, compute=pl.BF16, n_ctx=4096, max_batch=0):
    """A finalized model from a configuration and its tensors (name -> bf16 bit patterns or floats, [out, in])."""
    descs = layer_descs(config)
    m = LayerModel("pufivik", descs, n_embd=config["width"], n_vocab=config["vocab"], n_ctx=n_ctx, norm_eps=config["norm"]["eps"], compute=compute, logit_scale=1.0, max_batch=max_batch,
                   **model_opts(config))
    m.set_tensor(-1, "tok_embd", as_bf16(tensors["embed"]))
    m.set_tensor(-1, "output", as_bf16(tensors["embed"]))
    m.set_tensor(-1, "output_norm", as_f32(tensors["final.norm"]))
    first = next((i for i, d in enumerate(descs) if d["value_mix"]), None)
    for i, d in enumerate(descs):
        for role, a in layer_tensors(d, tensors, i, i == first):
            m.set_tensor(i, role, a)
    m.finalize()
    m.release_host()
    return m
