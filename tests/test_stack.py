"""CPU checks around models described layer by layer (Nevurax, Paposun): which model a folder holds, what of its config.json is refused, and
the oracle's own recurrences against closed forms."""
import copy
import ctypes
import json

import numpy as np
import pytest

from llm_metal_amd import lib
from llm_metal_amd.configs import GEMMA3, NEVURAX, PAPOSUN, QWEN3
from oracle import stack_oracle as so
from tests.stack_models import MODELS, Model


@pytest.fixture(scope="module")
def L():
    import os
    if not os.path.exists(lib.LIB_PATH):
        lib.build()
    return lib.load()


def test_which_model_a_folder_holds(L, tmp_path):
    def detect(text):
        (tmp_path / "config.json").write_text(text)
        return L.model_type_detect(str(tmp_path).encode())
    assert detect(json.dumps(MODELS["mixed"][0])) == NEVURAX
    assert detect(json.dumps(MODELS["norms around, mixed"][0])) == PAPOSUN
    assert detect('{"model_type": "qwen3"}') == QWEN3
    assert detect('{"model_type": "gemma3_text"}') == GEMMA3
    assert detect('not json, but "gemma3') == GEMMA3
    assert detect('{"architecture": "SomethingElse"}') == QWEN3
    assert L.model_type_detect(str(tmp_path / "model.safetensors").encode()) == QWEN3      # next to a file
    assert L.model_type_name(NEVURAX) == b"Nevurax" and L.model_type_name(PAPOSUN) == b"Paposun"
    assert [L.model_type_layered(t) for t in (QWEN3, GEMMA3, NEVURAX, PAPOSUN)] == [0, 0, 1, 1]


def test_config_errors_are_named(L, tmp_path, capfd):
    """A description that cannot be run is refused before anything touches a device, with the reason."""
    good = MODELS["mixed"][0]

    def refused(change, word):
        cfg = copy.deepcopy(good)
        change(cfg)
        (tmp_path / "config.json").write_text(json.dumps(cfg))
        assert not L.inference_state_create_from_file(str(tmp_path).encode(), NEVURAX, 64, 1)
        ctypes.CDLL(None).fflush(None)
        assert word in capfd.readouterr().err

    refused(lambda c: c.pop("vocab"), "vocab")
    refused(lambda c: c.pop("norm"), "eps")
    refused(lambda c: c.update(layers=[]), "layers")
    refused(lambda c: c["layers"][1].update(type="other"), "unknown mixer 'other'")
    refused(lambda c: c["layers"][0]["mlp"].update(kind="dense"), "unknown feed-forward 'dense'")
    refused(lambda c: c["layers"][1]["mixer"].pop("conv"), "layer 1: 'conv'")
    refused(lambda c: c["layers"][1]["mixer"].update(kv_heads=3), "multiple")
    refused(lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "'size'")
    refused(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "rot.dims")
    refused(lambda c: c["layers"][0]["mlp"]["router"].update(top=8), "'top'")
    (tmp_path / "config.json").write_text('{"vocab": 3,')
    assert not L.inference_state_create_from_file(str(tmp_path).encode(), NEVURAX, 64, 1)
    assert not L.inference_state_create_from_file(str(tmp_path).encode(), NEVURAX, 64, 0)   # no Q8_0 form


def test_config_errors_of_norms_around_are_named(L, tmp_path, capfd):
    good = MODELS["norms around, mixed"][0]

    def refused(change, word):
        cfg = copy.deepcopy(good)
        change(cfg)
        (tmp_path / "config.json").write_text(json.dumps(cfg))
        assert not L.inference_state_create_from_file(str(tmp_path).encode(), PAPOSUN, 64, 2)
        ctypes.CDLL(None).fflush(None)
        assert word in capfd.readouterr().err

    mixer = lambda c, i: c["layers"][i]["mixer"]
    refused(lambda c: c.pop("residual_mult"), "residual_mult")
    refused(lambda c: c.pop("logit_scale"), "logit_scale")
    refused(lambda c: c["layers"][1].update(type="delta"), "unknown mixer 'delta'")
    refused(lambda c: c["layers"][0]["mlp"].update(kind="moe"), "unknown feed-forward 'moe'")
    refused(lambda c: c["layers"][0]["mlp"].pop("ff"), "layer 0: 'ff'")
    refused(lambda c: mixer(c, 0)["mask"].update(size=0), "'size'")
    refused(lambda c: mixer(c, 0).update(kv_heads=4), "multiple")
    refused(lambda c: mixer(c, 0)["rot"].update(dims=26), "rot.dims")
    refused(lambda c: mixer(c, 0)["rot"]["scaling"].pop("low"), "'low'")
    refused(lambda c: mixer(c, 1).pop("gate_cap"), "gate_cap")
    refused(lambda c: mixer(c, 2).update(kv_from=1), "kv_from")
    refused(lambda c: mixer(c, 2).update(kv_from=2), "kv_from")
    refused(lambda c: mixer(c, 2)["rot"].update(base=3.0), "another rotation")
    refused(lambda c: mixer(c, 2).update(heads=4), "other heads")


def test_oracle_mlstm_is_the_sum_over_its_past():
    """The recurrence with its running maximum against the gated sum written out."""
    rng = np.random.default_rng(3)
    n, d, dv = 12, 5, 4
    q, k, v = rng.standard_normal((n, d)), rng.standard_normal((n, d)), rng.standard_normal((n, dv))
    i, f = rng.uniform(-6, 6, n), -rng.uniform(0, 3, n)
    S, N, m = np.zeros((d, dv)), np.zeros(d), 0.0
    for t in range(n):
        S, N, m, o = so.mlstm_step(S, N, m, q[t], k[t], v[t], i[t], f[t])
        w = np.array([np.exp(f[j + 1:t + 1].sum() + i[j]) * (k[j] @ q[t]) for j in range(t + 1)])
        peak = max([f[:t + 1].sum()] + [f[j + 1:t + 1].sum() + i[j] for j in range(t + 1)])     # what the sum is scaled by
        assert np.isclose(m, peak)
        assert np.allclose(o, (w @ v[:t + 1]) / (max(abs(w.sum()), 1.0) + 1e-6 * np.exp(peak)))


def test_oracle_frequencies():
    rot = {"dims": 8, "base": 10.0, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 2 * np.pi * 10}}
    plain = np.array([10.0 ** (-i / 4) for i in range(4)])           # turns within the original context: 10, 5.6, 3.2, 1.8
    got = np.array(so.scaled_frequencies(rot))
    assert np.allclose(got[:2], plain[:2])
    for j in (2, 3):
        mix = (10 * plain[j] - 1.0) / 3.0
        assert np.isclose(got[j], plain[j] * (mix + (1 - mix) / 4))
    rot["scaling"]["original"] /= 20
    assert np.allclose(so.scaled_frequencies(rot), plain / 4)        # every wavelength beyond the original context
    rng = np.random.default_rng(2)
    q, k = rng.standard_normal(10), rng.standard_normal(10)
    dots = [so.rotate_halves(q, p + 5, rot) @ so.rotate_halves(k, p, rot) for p in (0, 3, 40)]
    assert np.allclose(dots, dots[0]) and np.allclose(so.rotate_halves(q, 9, rot)[8:], q[8:])


def test_oracle_chunks(tmp_path):
    """A query sees its chunk: nothing before its first position, everything from there on."""
    cfg = MODELS["chunks, five heads, odd"][0]                           # chunks of 11
    m = Model(cfg, tmp_path)
    toks = m.tokens(30)
    full = so.run(cfg, m.W, toks)[-1]
    for at, same in ((21, True), (22, False), (0, True)):
        changed = list(toks)
        changed[at] = (toks[at] + 1) % cfg["vocab"]
        assert np.array_equal(so.run(cfg, m.W, changed)[-1], full) == same


def test_oracle_short_convolution_is_a_convolution():
    rng = np.random.default_rng(0)
    x, w = rng.standard_normal((9, 3)), rng.standard_normal((3, 4))
    state, got = {}, []
    for t in range(9):
        got.append(so.short_conv(state, "q", x[t], w))
    for c in range(3):
        assert np.allclose(np.convolve(x[:, c], w[c, ::-1])[:9], np.array(got)[:, c])


def test_oracle_delta_rule_recalls_a_key():
    """With no decay and full writes the state answers a unit key with the value last written under it."""
    rng = np.random.default_rng(1)
    S = np.zeros((8, 5))
    keys = np.linalg.qr(rng.standard_normal((8, 8)))[0]
    vals = rng.standard_normal((8, 5))
    for k, v in zip(keys, vals):
        S, o = so.delta_step(S, k, k, v, 1.0, 1.0)
        assert np.allclose(o, v)
    S, o = so.delta_step(S, keys[2], keys[2], 2 * vals[2], 1.0, 1.0)       # overwritten, the others kept
    assert np.allclose(o, 2 * vals[2]) and np.allclose(S.T @ keys[5], vals[5])
    S2, _ = so.delta_step(S, keys[0], keys[0], vals[0], np.full(8, 0.5), 0.0)
    assert np.allclose(S2, 0.5 * S)


def test_oracle_rotation_depends_on_distance_only():
    rng = np.random.default_rng(2)
    q, k = rng.standard_normal(8), rng.standard_normal(8)
    dots = [so.rotate_interleaved(q, p + 5, 8, 100.0) @ so.rotate_interleaved(k, p, 8, 100.0) for p in (0, 3, 40)]
    assert np.allclose(dots, dots[0])
    assert np.allclose(so.rotate_interleaved(q, 9, 4, 100.0)[4:], q[4:])


def test_oracle_attention_window(tmp_path):
    """A window of n sees n keys: the state of a model cut to the last n tokens gives the same layer output."""
    cfg, ra, rg = MODELS["latent, five heads, odd"]
    m = Model(cfg, tmp_path, ra, rg)
    toks = m.tokens(30)
    full = so.run(cfg, m.W, toks)[-1]
    changed = list(toks)
    changed[30 - 12] = (toks[30 - 12] + 1) % cfg["vocab"]                    # window 11: positions 19 .. 29
    assert np.array_equal(so.run(cfg, m.W, changed)[-1], full)
    changed = list(toks)
    changed[30 - 11] = (toks[30 - 11] + 1) % cfg["vocab"]
    assert not np.allclose(so.run(cfg, m.W, changed)[-1], full)
