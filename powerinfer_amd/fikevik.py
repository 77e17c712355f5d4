"""Fikevik: a decoder of gated linear attention layers (a decay per key channel) and layers in which windowed grouped-query attention and a matrix
memory with exponential gates work side by side; every sublayer's result is gated by its input and the norm comes after the residual sum; layers
may share their weights.  This module reads its configuration into layer descriptions (pi_model_create_layers) and its tensors into the
engine's roles; the computation is the engine's."""
import numpy as np

from . import lib as pl
from .checkpoint import as_bf16, as_f32
from .model import LayerModel

NO_LIMIT = float("inf")    # the feed-forward's GLU is not clamped
SILU_GAIN = 1.0


def owner(layers, i):
    """The layer whose tensors layer i uses."""
    seen = set()
    while layers[i].get("weights_of") is not None:
        if i in seen or not 0 <= layers[i]["weights_of"] < len(layers):
            raise ValueError(f"layer {i}: weights_of leads to no layer with weights of its own")
        seen.add(i)
        i = layers[i]["weights_of"]
    return i


def layer_descs(config, tensors):
    """tensors: for the sizes that only a tensor's shape gives."""
    out, layers = [], config["layers"]
    for i, layer in enumerate(layers):
        own, m, f = owner(layers, i), layer["mixer"], layer.get("mlp")
        d = dict(kv_from=-1, gated_residual=1, weights_of=0 if own == i else own + 1)
        if layer["type"] == "gla":
            d.update(mixer=pl.MIXER_KEYED, n_head=m["heads"], dim=m["dim"], vdim=m["vdim"], decay_tau=m["tau"], decay_rank=tensors[f"l{own}.mix.a1"].shape[0])
        elif layer["type"] == "parallel":
            a, r = m["left"], m["right"]
            rot, mask = a.get("rot") or {"dims": 0, "base": 1.0}, a.get("mask") or {"size": 0}
            d.update(mixer=pl.MIXER_GROUPED, n_head=a["heads"], n_kv_head=a["kv_heads"], dim=a["dim"], vdim=a["vdim"], rot_dim=rot["dims"], rot_base=rot["base"], rot_pairs=1,
                     scale=a["scale"], window=mask["size"], qk_norm=1, unit_v=1, head_temp=1, sink=-NO_LIMIT, out_scale=m["left_scale"],
                     mem_heads=r["heads"], mem_dim=r["dim"], mem_vdim=r["vdim"], mem_cap=r["gate_cap"], mem_scale=m["right_scale"])
        else:
            raise ValueError(f"layer {i}: mixer {layer['type']!r} is not part of this design")
        if f is None:
            d["ffn"] = pl.FFN_NONE
        elif f["kind"] == "dense":
            d.update(ffn=pl.FFN_GLU, glu_ff=f["ff"], glu_limit=NO_LIMIT, glu_gain=SILU_GAIN, glu_plain_up=1)
        else:
            raise ValueError(f"layer {i}: feed-forward {f['kind']!r} is not part of this design")
        out.append(d)
    return out


def model_opts(config):
    return dict(embed_scale=config["embedding"]["scale"], post_norm=1, residual_alpha=config["postln_alpha"])


def layer_tensors(d, t, i):
    """(role, array) of a layer with weights of its own."""
    p, bf, f32 = f"l{i}.", as_bf16, as_f32
    yield "attn_norm", f32(t[p + "norm1"])
    yield "res_gate", bf(t[p + "rg1"])
    yield "res_gate_b", f32(t[p + "rg1.b"])
    if d["mixer"] == pl.MIXER_KEYED:
        x = p + "mix."
        for role in ("q", "k", "v", "g", "a1", "a2"):
            yield "mix_" + role, bf(t[x + role])
        yield "mix_a2_b", f32(t[x + "a2.b"])
        yield "mix_norm", np.tile(f32(t[x + "norm"]), d["n_head"])                # one weight for all heads
        yield "wo", bf(t[x + "o"])
    else:
        x = p + "mix.left."
        for role in ("q", "k", "v"):
            yield "mix_" + role, bf(t[x + role])
        yield "mix_q_norm", f32(t[x + "q.norm"])
        yield "mix_k_norm", f32(t[x + "k.norm"])
        yield "mix_temp", f32(t[x + "temp"])
        yield "wo", bf(t[x + "o"])
        x = p + "mix.right."
        for role in ("q", "k", "v", "g", "o", "i", "f"):
            yield "mem_" + role, bf(t[x + role])
        for role in ("i", "f"):
            yield f"mem_{role}_b", f32(t[f"{x}{role}.b"])
        yield "mem_norm", f32(t[x + "norm"])
    if d["ffn"] == pl.FFN_GLU:
        yield "ffn_norm", f32(t[p + "norm2"])
        yield "res_gate_ffn", bf(t[p + "rg2"])
        yield "res_gate_ffn_b", f32(t[p + "rg2.b"])
        for role in ("gate", "up", "down"):
            yield "glu_" + role, bf(t[p + "mlp." + role])


def build(config, tensors, compute=pl.BF16, n_ctx=4096, max_batch=0):
    """A finalized model from a configuration and its tensors (name -> bf16 bit patterns or floats, [out, in])."""
    descs = layer_descs(config, tensors)
    m = LayerModel("fikevik", descs, n_embd=config["width"], n_vocab=config["vocab"], n_ctx=n_ctx, norm_eps=config["norm"]["eps"], compute=compute, max_batch=max_batch, **model_opts(config))
    m.set_tensor(-1, "tok_embd", as_bf16(tensors["embed"]))
    m.set_tensor(-1, "output_norm", as_f32(tensors["final.norm"]))
    m.set_tensor(-1, "output", as_bf16(tensors["head"]))
    for i, d in enumerate(descs):
        if not d["weights_of"]:
            for role, a in layer_tensors(d, tensors, i):
                m.set_tensor(i, role, a)
    m.finalize()
    m.release_host()
    return m
