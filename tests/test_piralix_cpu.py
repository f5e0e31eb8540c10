"""Piralix without a GPU: the plain implementation's own consistency, registry, configuration."""
import json

import numpy as np
import pytest

import piralix_plain as plain
from piralix_cases import SPECS, STRETCH, random_tensors
from ritevik_cases import bf16_bits


def test_rotation_turns_neighbours_and_keeps_the_rest():
    x = np.random.default_rng(0).standard_normal((5, 2, 10))
    y = plain.rotate_pairs(x, np.arange(5), dict(dims=6, base=100.0))
    assert np.allclose(y[0], x[0]) and np.array_equal(y[..., 6:], x[..., 6:])
    for i in range(3):
        z = (x[4, :, 2 * i] + 1j * x[4, :, 2 * i + 1]) * np.exp(4j * 100.0 ** (-2 * i / 6))
        assert np.allclose(y[4, :, 2 * i], z.real) and np.allclose(y[4, :, 2 * i + 1], z.imag)


def test_stretched_frequencies():
    """Fast pairs keep their frequency, slow ones are divided by the factor, the ramp lies between; a ramp of no width is a step."""
    rot = dict(dims=48, base=20000.0, scaling=dict(factor=6.0, fast=20.0, slow=2.0, original=3000))
    f, grow = plain.frequencies(rot)
    f0, one = plain.frequencies(dict(dims=48, base=20000.0))
    assert one == 1.0 and np.isclose(grow, 0.1 * np.log(6.0) + 1.0)
    assert np.allclose(f[:5], f0[:5]) and np.allclose(f[-3:], f0[-3:] / 6.0) and (np.diff(f0 / f) >= 0).all()
    turns = 3000 * f0 / (2 * np.pi)  # over the original positions
    assert np.allclose(f[turns > 40], f0[turns > 40]) and np.allclose(f[turns < 1], f0[turns < 1] / 6.0) and ((f0 / f > 1.01) & (f0 / f < 5.99)).any()
    narrow, _ = plain.frequencies(dict(dims=48, base=20000.0, scaling=dict(factor=6.0, fast=1e9, slow=1e9, original=64)))
    assert np.allclose(f0[1:] / narrow[1:], 6.0) and np.isclose(f0[0], narrow[0])


def test_memory_reads_back_what_was_written():
    """With gates that neither forget nor scale, the read-out of a unit key is the value written under it over its count."""
    T, D, DV = 3, 3, 2
    k = np.eye(D)[[0, 1, 0]].reshape(T, 1, D)
    v = np.random.default_rng(1).standard_normal((T, 1, DV))
    o = plain.matrix_memory_recurrence(k, k, v, np.zeros((T, 1)), np.zeros((T, 1)))
    assert np.allclose(o[:2], v[:2], atol=1e-5) and np.allclose(o[2], (v[0] + v[2]) / 2, atol=1e-5)
    # the running maximum starts at zero: a weak input gate stays weak under the floor of the denominator
    weak = plain.matrix_memory_recurrence(k[:1], k[:1], v[:1], np.full((1, 1), -5.0), np.zeros((1, 1)))
    assert np.allclose(weak, v[:1] * np.exp(-5.0), rtol=1e-5)


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


def test_registry_and_configuration(agpu, tmp_path):
    from async_gpu_amd import _lib, models, piralix, weights
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Piralix"}))
    assert models.architecture(str(tmp_path)) == "Piralix"
    s = SPECS["mixed"]
    cfg = piralix.PiralixConfig(s, n_positions=33, max_batch=2, dtype="float32")
    st, layers = cfg.struct(), cfg.layer_structs()
    assert (st.n_layer, st.width, st.vocab_size, st.n_positions, st.max_batch) == (6, 100, 131, 33, 2)
    assert (st.loop_start, st.loop_stop, st.loop_times, st.dtype) == (1, 4, 3, _lib.DTYPE_F32)
    a = layers[0]
    assert a.mixer == _lib.MIXER_GROUPED_ATTENTION and (a.heads, a.kv_heads, a.dim, a.vdim, a.rot_dims, a.ff) == (6, 2, 24, 40, 16, 80)
    assert (a.rot_base, a.rot_factor, a.rot_original, a.rot_fast, a.rot_slow) == (5000.0, STRETCH["factor"], STRETCH["original"], STRETCH["fast"], STRETCH["slow"])
    assert a.softcap == 20.0 and np.isclose(a.ff_limit, 1.3)
    assert layers[1].mixer == _lib.MIXER_MATRIX_MEMORY and layers[1].gate_cap == 9.0 and np.isclose(layers[1].ff_limit, 0.8)
    assert layers[2].mixer == _lib.MIXER_GATED_LRU and (layers[2].lru_width, layers[2].blocks, layers[2].conv, layers[2].ff) == (84, 3, 4, 0)
    none = piralix.PiralixConfig(SPECS["plain"])
    assert none.struct().loop_times == 0 and none.layer_structs()[2].rot_factor == 0.0
    with pytest.raises(ValueError):
        piralix.PiralixConfig(s, dtype="float16")
    for change in (lambda e: e.update(type="something"), lambda e: e["mlp"].update(kind="sparse")):
        bad = json.loads(json.dumps(s))
        change(bad["layers"][0])
        with pytest.raises(weights.ModelFileError):
            piralix.PiralixConfig(bad).layer_structs()
    assert piralix.PiralixModel._rows_cols((3, 5, 7)) == (15, 7) and piralix.PiralixModel._rows_cols((4,)) == (1, 4)
    assert bf16_bits(np.float32(1.0)) == 0x3F80
