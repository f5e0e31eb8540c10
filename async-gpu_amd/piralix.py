"""Piralix over the model-level C ABI (include/agpu_piralix.h): configuration, model."""
from . import _lib, weights
from .layered import DTYPES, LayeredConfig, LayeredModel


class PiralixConfig(LayeredConfig):
    def struct(self):
        return _lib.PiralixConfigStruct(self.n_layer, self.width, self.vocab_size, self.n_positions, self.max_batch,
                                        float(self.spec["norm"]["eps"]), *self.loop, DTYPES[self.dtype], int(self.argmax_last))

    def layer_structs(self):
        out = (_lib.PiralixLayerStruct * self.n_layer)()
        for i, entry in enumerate(self.spec["layers"]):
            mix, mlp, s = entry["mixer"], self.dense_ff(entry, i), out[i]
            if mlp:
                s.ff, s.ff_limit = int(mlp["ff"]), float(mlp["limit"])
            if entry["type"] == "mlstm":
                s.mixer = _lib.MIXER_MATRIX_MEMORY
                s.heads, s.dim, s.vdim, s.gate_cap = int(mix["heads"]), int(mix["dim"]), int(mix["vdim"]), float(mix["gate_cap"])
            elif entry["type"] == "attention":
                s.mixer = _lib.MIXER_GROUPED_ATTENTION
                s.heads, s.kv_heads, s.dim, s.vdim = (int(mix[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
                s.scale, s.softcap = float(mix["scale"]), float(mix.get("softcap") or 0.0)
                rot = mix.get("rot") or {}
                s.rot_dims, s.rot_base = int(rot.get("dims", 0)), float(rot.get("base", 10000.0))
                stretch = rot.get("scaling")
                if stretch:
                    s.rot_factor, s.rot_original, s.rot_fast, s.rot_slow = (float(stretch[k]) for k in ("factor", "original", "fast", "slow"))
            elif entry["type"] == "rglru":
                s.mixer = _lib.MIXER_GATED_LRU
                s.lru_width, s.blocks, s.conv = int(mix["width"]), int(mix["blocks"]), int(mix["conv"])
            else:
                raise weights.ModelFileError(f"layer {i}: mixer type {entry['type']!r} is not known")
        return out


class PiralixModel(LayeredModel):
    prefix = "agpu_piralix"

    @classmethod
    def make_config(cls, spec, shape_of, **config_kw):
        return PiralixConfig(spec, **config_kw)
