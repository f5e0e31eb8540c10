"""Ritevik over the model-level C ABI (include/agpu_ritevik.h): configuration, weight loading, model."""
import ctypes as C
import json
import os

import numpy as np

from . import _lib, weights
from .language_model import LanguageModel, _np

DTYPES = {"bfloat16": _lib.DTYPE_BF16, "float32": _lib.DTYPE_F32}


class RitevikConfig:
    """A model's config.json (`spec`: the parsed dictionary) plus what the caller chooses: positions the cache holds, batch,
    number format, tie rule.  The low-rank sizes of delta layers come from the weights' shapes (`ranks`: per layer
    (decay, gate) or None)."""

    def __init__(self, spec, ranks, n_positions=1024, max_batch=1, dtype="bfloat16", argmax_last=False):
        if dtype not in DTYPES:
            raise ValueError(f"dtype {dtype!r} is not one of {sorted(DTYPES)}")
        self.spec, self.ranks = spec, ranks
        self.n_positions, self.max_batch, self.dtype, self.argmax_last = int(n_positions), int(max_batch), dtype, argmax_last
        self.vocab_size, self.width = int(spec["vocab"]), int(spec["width"])
        self.n_layer = len(spec["layers"])

    def struct(self):
        loop = self.spec.get("loop") or {}
        side = self.spec.get("token_side") or {}
        return _lib.RitevikConfigStruct(
            self.n_layer, self.width, self.vocab_size, self.n_positions, self.max_batch, float(self.spec["norm"]["eps"]),
            int(loop.get("start", 0)), int(loop.get("stop", 0)), int(loop.get("times", 0)), int(side.get("dim", 0)),
            DTYPES[self.dtype], int(self.argmax_last))

    def layer_structs(self):
        out = (_lib.RitevikLayerStruct * self.n_layer)()
        for i, entry in enumerate(self.spec["layers"]):
            mix, mlp, s = entry["mixer"], entry.get("mlp"), out[i]
            s.heads, s.dim, s.vdim = int(mix["heads"]), int(mix["dim"]), int(mix["vdim"])
            if mlp:
                if mlp.get("kind") != "dense":
                    raise weights.ModelFileError(f"layer {i}: feed-forward kind {mlp.get('kind')!r} is not known")
                s.ff = int(mlp["ff"])
            if entry["type"] == "latent_attention":
                s.mixer = _lib.MIXER_LATENT_ATTENTION
                s.kv_rank, s.rot_dim, s.rot_dims = int(mix["kv_rank"]), int(mix["rot_dim"]), int(mix["rot"]["dims"])
                s.scale, s.rot_base = float(mix["scale"]), float(mix["rot"]["base"])
            elif entry["type"] == "channel_delta":
                s.mixer = _lib.MIXER_CHANNEL_DELTA
                s.kv_heads, s.conv = int(mix["kv_heads"]), int(mix["conv"])
                s.decay_rank, s.gate_rank = self.ranks[i]
            else:
                raise weights.ModelFileError(f"layer {i}: mixer type {entry['type']!r} is not known")
        return out


def delta_ranks(spec, shape_of):
    """Per layer (decay rank, gate rank) read off the shapes of the first low-rank factors, None for other layers."""
    return [(int(shape_of(f"l{i}.mix.a1")[0]), int(shape_of(f"l{i}.mix.g1")[0])) if e["type"] == "channel_delta" else None
            for i, e in enumerate(spec["layers"])]


class RitevikModel(LanguageModel):
    """Device-resident Ritevik.  `ctx` must own its stream, as for Int4Gpt2Model."""

    prefix = "agpu_ritevik"

    def __init__(self, config, ctx=None, device=0):
        self.config = config
        self.ctx = ctx if ctx is not None else _lib.Context(device)
        self._lib = _lib.cdll()
        h = C.c_void_p()
        st, layers = config.struct(), config.layer_structs()
        self._check(self._lib.agpu_ritevik_create(self.ctx.handle, C.addressof(st), C.addressof(layers), C.byref(h)))
        self.handle = h

    @classmethod
    def from_tensors(cls, spec, tensors, ctx=None, device=0, **config_kw):
        """tensors: {name: (dtype, array)} as weights.read_safetensors returns it."""
        def shape_of(name):
            if name not in tensors:
                raise weights.ModelFileError(f"tensor '{name}' not found")
            return tensors[name][1].shape
        m = cls(RitevikConfig(spec, delta_ranks(spec, shape_of), **config_kw), ctx, device)
        for name, rows, cols, _ in m.tensor_list():
            shape = shape_of(name)
            dtype, a = tensors[name]
            if len(shape) == 1:
                shape = (1, shape[0])
            if tuple(shape) != (rows, cols):
                raise weights.ModelFileError(f"tensor '{name}': expected shape {[rows, cols]}, got {list(shape)}")
            if dtype not in ("BF16", "F32"):
                raise weights.ModelFileError(f"tensor '{name}': expected dtype BF16 or F32, got {dtype}")
            m.set_tensor(name, a)
        return m

    @classmethod
    def from_directory(cls, path, ctx=None, device=0, **config_kw):
        """A folder with config.json and model.safetensors."""
        with open(os.path.join(path, "config.json")) as f:
            spec = json.load(f)
        return cls.from_tensors(spec, weights.read_safetensors(os.path.join(path, "model.safetensors")), ctx, device, **config_kw)

    def tensor_list(self):
        """[(name, rows, cols, is set)] of every tensor this configuration needs."""
        out, i = [], 0
        name, rows, cols, is_set = C.c_char_p(), C.c_int64(0), C.c_int64(0), C.c_int32(0)
        while self._lib.agpu_ritevik_tensor_info(self.handle, i, C.byref(name), C.addressof(rows), C.addressof(cols), C.addressof(is_set)) == 0:
            out.append((name.value.decode(), int(rows.value), int(cols.value), bool(is_set.value)))
            i += 1
        return out

    def set_tensor(self, name, a):
        """uint16 arrays are bf16 bits, everything else goes as float32."""
        if a.dtype == np.uint16:
            a, dtype = _np(a, np.uint16), _lib.DTYPE_BF16
        else:
            a, dtype = _np(a, np.float32), _lib.DTYPE_F32
        rows, cols = (1, a.shape[0]) if a.ndim == 1 else a.shape
        self._call("agpu_ritevik_set_tensor", name.encode(), a, dtype, rows, cols)

    def weight_bytes(self):
        return int(self._lib.agpu_ritevik_weight_bytes(self.handle))

    def cache_bytes(self):
        return int(self._lib.agpu_ritevik_cache_bytes(self.handle))

    def layer_runs(self):
        return int(self._lib.agpu_ritevik_layer_runs(self.handle))

    def layer_streams(self, tokens):
        """Feeds `tokens` to the cached sequence and returns the residual stream after every layer run, [runs, tokens, width]."""
        tokens = _np(tokens, np.uint32).ravel()
        out = np.empty((self.layer_runs(), tokens.size, self.config.width), np.float32)
        p = self.ctx.upload(tokens)
        try:
            self._call("agpu_ritevik_layer_streams", p, tokens.size, out)
        finally:
            self.ctx.free(p)
        return out
