"""Ritevik without a GPU: the plain implementation's own consistency, weight files, registry, configuration."""
import json

import numpy as np
import pytest

import ritevik_plain as plain
from ritevik_cases import SPECS, bf16_bits, bf16_values, random_tensors


def test_rotation_turns_pairs_and_keeps_the_rest():
    x = np.random.default_rng(0).standard_normal((5, 2, 10))
    y = plain.rotate_half(x, np.arange(5), 6, 100.0)
    assert np.allclose(y[0], x[0]) and np.array_equal(y[..., 6:], x[..., 6:])
    for i in range(3):
        a = 4 * 100.0 ** (-2 * i / 6)
        z = (x[4, :, i] + 1j * x[4, :, i + 3]) * np.exp(1j * a)
        assert np.allclose(y[4, :, i], z.real) and np.allclose(y[4, :, i + 3], z.imag)


def test_delta_recurrence_is_the_delta_rule():
    """Without decay and with beta 1 a unit key reads back exactly what was written under it last."""
    rng = np.random.default_rng(1)
    T, D, DV = 4, 4, 3
    k = np.eye(D)[[0, 1, 2, 1]].reshape(T, 1, D)
    v = rng.standard_normal((T, 1, DV))
    o, S = plain.delta_recurrence(k, k, v, np.ones((T, 1, D)), np.ones((T, 1)))
    assert np.allclose(o, v) and np.allclose(S[0, 1], v[3, 0]) and np.allclose(S[0, 0], v[0, 0]) and not S[0, 3].any()
    # a decay acts on rows of S that belong to key channels, before the write
    g = np.ones((T, 1, D))
    g[3, 0, 0] = 0.25
    _, S2 = plain.delta_recurrence(k, k, v, g, np.ones((T, 1)))
    assert np.allclose(S2[0, 0], 0.25 * v[0, 0]) and np.allclose(S2[0, 1:], S[0, 1:])


@pytest.mark.parametrize("name", sorted(SPECS))
def test_plain_model_is_causal(name):
    s = SPECS[name]
    _, w = random_tensors(s, 1)
    t = np.random.default_rng(2).integers(0, s["vocab"], 20)
    a = plain.forward(t, s, w)
    t2 = t.copy()
    t2[12:] = (t2[12:] + 1) % s["vocab"]
    b = plain.forward(t2, s, w)
    assert np.allclose(a[:12], b[:12]) and not np.allclose(a[12], b[12])


def test_bf16_rounding(agpu):
    from async_gpu_amd import weights
    x = np.array([1.0, 1.00390625, 1.001953125, 1.005859375, -3.1415927, 0.0, 1e-30], np.float32)
    assert np.array_equal(weights.f32_to_bf16(x), bf16_bits(x))
    assert np.array_equal(weights.bf16_to_f32(weights.f32_to_bf16(x)).astype(np.float64), bf16_values(bf16_bits(x)))
    assert bf16_values(bf16_bits(x))[1] == 1.0 and bf16_values(bf16_bits(x))[3] == 1.0078125  # ties to even


def test_safetensors_round_trip(agpu, tmp_path):
    from async_gpu_amd import weights
    path = str(tmp_path / "x.safetensors")
    t = {"a": ("BF16", np.arange(6, dtype=np.uint16).reshape(2, 3)), "b.c": ("F32", np.linspace(0, 1, 4, dtype=np.float32)),
         "i": ("I32", np.array([[-1], [7]], np.int32))}
    weights.write_safetensors(path, t)
    got = weights.read_safetensors(path)
    assert set(got) == set(t)
    for k in t:
        assert got[k][0] == t[k][0] and np.array_equal(got[k][1], t[k][1]) and got[k][1].shape == t[k][1].shape
    from safetensors import safe_open
    with safe_open(path, framework="numpy") as f:
        assert np.array_equal(f.get_tensor("b.c"), t["b.c"][1])
    raw = open(path, "rb").read()
    bad = str(tmp_path / "bad.safetensors")
    open(bad, "wb").write(raw[:-4])
    with pytest.raises(weights.ModelFileError):
        weights.read_safetensors(bad)


def test_registry_picks_the_architecture(agpu, tmp_path):
    from async_gpu_amd import models, weights
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Ritevik"}))
    assert models.architecture(str(tmp_path)) == "Ritevik"
    (tmp_path / "config.json").write_text(json.dumps({"architectures": ["GPT2LMHeadModel"]}))
    assert models.architecture(str(tmp_path)) == "GPT2LMHeadModel"
    assert models.architecture(str(tmp_path / "model.safetensors")) == "GPT2LMHeadModel"
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Nobody"}))
    with pytest.raises(weights.ModelFileError, match="Nobody"):
        models.architecture(str(tmp_path))


def test_configuration_reaches_the_structs(agpu):
    from async_gpu_amd import _lib, ritevik, weights
    s = SPECS["mixed"]
    bits, _ = random_tensors(s, 1)
    ranks = ritevik.delta_ranks(s, lambda name: bits[name].shape)
    assert ranks == [None, (12, 20), (12, 20), None, (40, 8)]
    cfg = ritevik.RitevikConfig(s, ranks, n_positions=33, max_batch=2, dtype="float32")
    st, layers = cfg.struct(), cfg.layer_structs()
    assert (st.n_layer, st.width, st.vocab_size, st.n_positions, st.max_batch) == (5, 100, 131, 33, 2)
    assert (st.loop_start, st.loop_stop, st.loop_times, st.side_dim, st.dtype) == (1, 4, 3, 12, _lib.DTYPE_F32)
    assert layers[0].mixer == _lib.MIXER_LATENT_ATTENTION and layers[0].rot_base == 10000.0 and layers[0].ff == 80
    assert layers[2].mixer == _lib.MIXER_CHANNEL_DELTA and layers[2].ff == 0 and layers[2].conv == 2
    assert (layers[4].kv_heads, layers[4].decay_rank, layers[4].gate_rank) == (1, 40, 8)
    none = ritevik.RitevikConfig(SPECS["plain"], [(7, 70), None]).struct()
    assert none.loop_times == 0 and none.side_dim == 0
    with pytest.raises(ValueError):
        ritevik.RitevikConfig(s, ranks, dtype="float16")
    bad = json.loads(json.dumps(s))
    bad["layers"][0]["type"] = "something"
    with pytest.raises(weights.ModelFileError):
        ritevik.RitevikConfig(bad, ranks).layer_structs()
