"""The model registry: picks the model class by what a path holds.

A folder with a config.json that names its architecture is loaded by that architecture's loader; a safetensors file (or a
folder with a model.safetensors and no architecture the registry knows by name) is a GPT-2 file, fp32 or int4."""
import json
import os

from . import weights


def _layered(model_class, path, dtype, n_positions, max_batch, ctx, device):
    return model_class.from_directory(path, ctx, device, dtype=dtype, n_positions=n_positions or 1024, max_batch=max_batch)


def _ritevik(*args):
    from .ritevik import RitevikModel
    return _layered(RitevikModel, *args)


def _piralix(*args):
    from .piralix import PiralixModel
    return _layered(PiralixModel, *args)


def _gpt2(path, dtype, n_positions, max_batch, ctx, device):
    # int4 weights, fp32 activations and cache whatever number format is asked for; the file fixes the positions
    from .gpt2 import Int4Gpt2Model
    if os.path.isdir(path):
        path = os.path.join(path, "model.safetensors")
    return Int4Gpt2Model.from_file(path, ctx=ctx, device=device, max_batch=max_batch)


ARCHITECTURES = {"Ritevik": _ritevik, "Piralix": _piralix, "GPT2LMHeadModel": _gpt2}


def architecture(path):
    """The registry's name of the model at `path`."""
    if os.path.isdir(path):
        config = os.path.join(path, "config.json")
        if os.path.exists(config):
            with open(config) as f:
                spec = json.load(f)
            name = spec.get("architecture") or (spec.get("architectures") or [None])[0]
            if name in ARCHITECTURES:
                return name
            if name is not None:
                raise weights.ModelFileError(f"{config}: architecture {name!r} is not one of {sorted(ARCHITECTURES)}")
    return "GPT2LMHeadModel"


def load_model(path, dtype="bfloat16", n_positions=None, max_batch=1, ctx=None, device=0):
    """The model at `path`.  dtype "bfloat16" or "float32": the number format of a model that has both; n_positions: the cache
    size of a model whose file does not fix it (default 1024)."""
    return ARCHITECTURES[architecture(path)](path, dtype, n_positions, max_batch, ctx, device)
