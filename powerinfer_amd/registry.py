"""Model registry: which loader serves a file or folder.

* a folder with config.json + model.safetensors: its "architecture" names the design (FOLDERS);
* a GGUF file: its general.architecture (llama, falcon) through powerinfer_amd.gguf.
"""
import os

from . import checkpoint, lib as pl

COMPUTE = {"bfloat16": pl.BF16, "float32": pl.F32}


def _lerasun(config, tensors, **kw):
    from . import lerasun
    return lerasun.build(config, tensors, **kw)


def _pibalorn(config, tensors, **kw):
    from . import pibalorn
    return pibalorn.build(config, tensors, **kw)


def _fikevik(config, tensors, **kw):
    from . import fikevik
    return fikevik.build(config, tensors, **kw)


def _pufivik(config, tensors, **kw):
    from . import pufivik
    return pufivik.build(config, tensors, **kw)


FOLDERS = {"Lerasun": _lerasun, "Pibalorn": _pibalorn, "Fikevik": _fikevik, "Pufivik": _pufivik}


def load_model(path, dtype="bfloat16", n_ctx=4096, max_batch=0):
    """A model ready to run.  dtype: bfloat16 (served precision) or float32, for designs described layer by layer; GGUF models run in
    the types their file holds."""
    if os.path.isdir(path):
        config = checkpoint.read_config(path)
        arch = config.get("architecture")
        if arch not in FOLDERS:
            raise ValueError(f"{path}: architecture {arch!r} is not registered (known: {', '.join(sorted(FOLDERS))})")
        tensors = checkpoint.read_safetensors(os.path.join(path, "model.safetensors"))
        return FOLDERS[arch](config, tensors, compute=COMPUTE[dtype], n_ctx=n_ctx, max_batch=max_batch)
    from . import gguf
    from .model import Model
    hp, model = gguf.read_model(path, n_ctx=n_ctx)
    return Model(hp).load(model)
