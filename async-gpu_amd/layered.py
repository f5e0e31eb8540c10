"""What the models with bf16 weights share on the Python side: loading a folder, named tensors, the residual stream behind every
layer run.  Their C entry points have the same names behind each model's prefix."""
import ctypes as C
import json
import os

import numpy as np

from . import _lib, weights
from .language_model import LanguageModel, _np

DTYPES = {"bfloat16": _lib.DTYPE_BF16, "float32": _lib.DTYPE_F32}


class LayeredConfig:
    """A model's config.json (`spec`: the parsed dictionary) plus what the caller chooses: positions the cache holds, batch,
    number format, tie rule."""

    def __init__(self, spec, n_positions=1024, max_batch=1, dtype="bfloat16", argmax_last=False):
        if dtype not in DTYPES:
            raise ValueError(f"dtype {dtype!r} is not one of {sorted(DTYPES)}")
        self.spec = spec
        self.n_positions, self.max_batch, self.dtype, self.argmax_last = int(n_positions), int(max_batch), dtype, argmax_last
        self.vocab_size, self.width = int(spec["vocab"]), int(spec["width"])
        self.n_layer = len(spec["layers"])
        loop = spec.get("loop") or {}
        self.loop = tuple(int(loop.get(k, 0)) for k in ("start", "stop", "times"))

    @staticmethod
    def dense_ff(entry, i):
        """The feed-forward of layer i, or None."""
        mlp = entry.get("mlp")
        if mlp and mlp.get("kind") != "dense":
            raise weights.ModelFileError(f"layer {i}: feed-forward kind {mlp.get('kind')!r} is not known")
        return mlp


class LayeredModel(LanguageModel):
    """Device-resident model of a LayeredConfig.  `ctx` must own its stream, as for Int4Gpt2Model."""

    def __init__(self, config, ctx=None, device=0):
        self.config = config
        self.ctx = ctx if ctx is not None else _lib.Context(device)
        self._lib = _lib.cdll()
        h = C.c_void_p()
        st, layers = config.struct(), config.layer_structs()
        self._check(self._entry("create")(self.ctx.handle, C.addressof(st), C.addressof(layers), C.byref(h)))
        self.handle = h

    def _entry(self, name):
        return getattr(self._lib, f"{self.prefix}_{name}")

    @classmethod
    def make_config(cls, spec, shape_of, **config_kw):
        """The configuration of a model whose tensors have the shapes that shape_of(name) tells."""
        raise NotImplementedError

    @classmethod
    def from_tensors(cls, spec, tensors, ctx=None, device=0, **config_kw):
        """tensors: {name: (dtype, array)} as weights.read_safetensors returns it."""
        def shape_of(name):
            if name not in tensors:
                raise weights.ModelFileError(f"tensor '{name}' not found")
            return tensors[name][1].shape
        m = cls(cls.make_config(spec, shape_of, **config_kw), ctx, device)
        for name, rows, cols, _ in m.tensor_list():
            shape = shape_of(name)
            dtype, a = tensors[name]
            if m._rows_cols(shape) != (rows, cols):
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

    @staticmethod
    def _rows_cols(shape):
        """A vector has one row, a tensor of three dimensions the first two as its rows."""
        return int(np.prod(shape[:-1], dtype=np.int64)), int(shape[-1])

    def tensor_list(self):
        """[(name, rows, cols, is set)] of every tensor this configuration needs."""
        out, i = [], 0
        name, rows, cols, is_set = C.c_char_p(), C.c_int64(0), C.c_int64(0), C.c_int32(0)
        while self._entry("tensor_info")(self.handle, i, C.byref(name), C.addressof(rows), C.addressof(cols), C.addressof(is_set)) == 0:
            out.append((name.value.decode(), int(rows.value), int(cols.value), bool(is_set.value)))
            i += 1
        return out

    def set_tensor(self, name, a):
        """uint16 arrays are bf16 bits, everything else goes as float32."""
        if a.dtype == np.uint16:
            a, dtype = _np(a, np.uint16), _lib.DTYPE_BF16
        else:
            a, dtype = _np(a, np.float32), _lib.DTYPE_F32
        rows, cols = self._rows_cols(a.shape)
        self._call(self.prefix + "_set_tensor", name.encode(), a, dtype, rows, cols)

    def weight_bytes(self):
        return int(self._entry("weight_bytes")(self.handle))

    def cache_bytes(self):
        return int(self._entry("cache_bytes")(self.handle))

    def layer_runs(self):
        return int(self._entry("layer_runs")(self.handle))

    def layer_streams(self, tokens):
        """Feeds `tokens` to the cached sequence and returns the residual stream after every layer run, [runs, tokens, width]."""
        tokens = _np(tokens, np.uint32).ravel()
        out = np.empty((self.layer_runs(), tokens.size, self.config.width), np.float32)
        p = self.ctx.upload(tokens)
        try:
            self._call(self.prefix + "_layer_streams", p, tokens.size, out)
        finally:
            self.ctx.free(p)
        return out
