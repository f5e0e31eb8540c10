"""Ritevik over the model-level C ABI (include/agpu_ritevik.h): configuration, model."""
from . import _lib, weights
from .layered import DTYPES, LayeredConfig, LayeredModel


class RitevikConfig(LayeredConfig):
    """The low-rank sizes of delta layers come from the weights' shapes (`ranks`: per layer (decay, gate) or None)."""

    def __init__(self, spec, ranks, **kw):
        super().__init__(spec, **kw)
        self.ranks = ranks

    def struct(self):
        side = self.spec.get("token_side") or {}
        return _lib.RitevikConfigStruct(
            self.n_layer, self.width, self.vocab_size, self.n_positions, self.max_batch, float(self.spec["norm"]["eps"]),
            *self.loop, int(side.get("dim", 0)),
            DTYPES[self.dtype], int(self.argmax_last))

    def layer_structs(self):
        out = (_lib.RitevikLayerStruct * self.n_layer)()
        for i, entry in enumerate(self.spec["layers"]):
            mix, mlp, s = entry["mixer"], self.dense_ff(entry, i), out[i]
            s.heads, s.dim, s.vdim = int(mix["heads"]), int(mix["dim"]), int(mix["vdim"])
            if mlp:
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


class RitevikModel(LayeredModel):
    prefix = "agpu_ritevik"

    @classmethod
    def make_config(cls, spec, shape_of, **config_kw):
        return RitevikConfig(spec, delta_ranks(spec, shape_of), **config_kw)
