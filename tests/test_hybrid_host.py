"""CPU side of the hybrid decoder: the plain implementation the GPU tests lean on (checked against itself where two of its ways must
agree), the model registry, and what the loader says about files that are not right."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from crabml_amd import synth_hybrid as sh
from tests import hybrid_oracle as ho

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
CONFIG = sh.config(40, 30, [sh.layer(4, 2, 8, 12, 5, 3, 6, 10, 24), sh.layer(2, 1, 10, 8, 9, 2, 8, 8, None)], loop={"start": 0, "stop": 1, "times": 2})


@pytest.fixture(scope="module")
def model():
    return {k: sh.from_bf16(v) for k, v in sh.random_tensors(CONFIG, 3).items()}


# ---- the oracle ---------------------------------------------------------------------------------------------------------------------------
def test_oracle_is_causal(model):
    t = [3, 1, 4, 1, 5, 9, 2, 6, 5, 3, 5, 8]
    full = ho.forward(CONFIG, model, t)
    for n in (1, 5, 6, 11):
        assert np.allclose(ho.forward(CONFIG, model, t[:n]), full[:n], rtol=0, atol=1e-10)


def test_oracle_attention_against_a_loop_over_keys():
    rng = np.random.default_rng(0)
    T, H, G, d, dv, chunk = 23, 6, 3, 5, 4, 7
    q, k, v = rng.standard_normal((T, H, d)), rng.standard_normal((T, G, d)), rng.standard_normal((T, G, dv))
    amp, rate, sink = rng.uniform(0, 2, H), rng.uniform(0, 1, H), rng.standard_normal(H)
    got = ho.softmax_attention(q, k, v, 0.4, chunk, amp, rate, sink)
    for i in range(T):
        for h in range(H):
            num, den = np.zeros(dv), np.exp(sink[h])
            for j in range((i // chunk) * chunk, i + 1):
                w = np.exp(q[i, h] @ k[j, h // 2] * 0.4 - amp[h] * np.log(1 + rate[h] * (i - j)))
                num, den = num + w * v[j, h // 2], den + w
            assert np.allclose(got[i, h], num / den, atol=1e-12)


def test_oracle_recurrence_against_its_sum():
    rng = np.random.default_rng(1)
    T, H, d, dv = 17, 2, 4, 3
    q, k, v = rng.standard_normal((T, H, d)), rng.standard_normal((T, H, d)), rng.standard_normal((T, H, dv))
    decay = [0.7, 1.0]
    got, state = ho.decaying_linear_attention(q, k, v, decay)
    for h in range(H):
        for t in range(T):
            want = sum(decay[h] ** (t - j) * (q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1))
            assert np.allclose(got[t, h], want, atol=1e-12)
    half, mid = ho.decaying_linear_attention(q[:8], k[:8], v[:8], decay)
    rest, end = ho.decaying_linear_attention(q[8:], k[8:], v[8:], decay, mid)
    assert np.allclose(np.concatenate([half, rest]), got) and np.allclose(end, state)


def test_oracle_activation_is_smooth_at_zero_and_bends_with_its_numbers():
    z = np.array([-1e-6, 0.0, 1e-6])
    y = ho.xielu(z, 0.3, -0.2)
    assert y[1] == 0 and np.allclose(np.diff(y), 0.5e-6, rtol=1e-4)
    assert np.isclose(ho.xielu(np.array([2.0]), 0.0, 0.0)[0], np.log(2) * 4 + 1)
    assert np.isclose(ho.xielu(np.array([-1.0]), 0.0, 0.0)[0], (0.5 + np.log(2)) * (np.exp(-1) - 1 + 1) - 0.5)


def test_oracle_loop_order():
    c = dict(CONFIG, layers=[CONFIG["layers"][1]] * 5, loop={"start": 1, "stop": 3, "times": 3})
    assert ho.run_order(c) == [(0, None, False), (1, 0, True), (2, 0, False), (1, 1, True), (2, 1, False), (1, 2, True), (2, 2, False), (3, None, False),
                               (4, None, False)]
    assert ho.run_order(dict(c, loop=None)) == [(i, None, False) for i in range(5)]


def test_bf16_conversion_rounds_to_even():
    x = np.array([1.0, 1.0 + 2 ** -8, 1.0 + 3 * 2 ** -8, -3.3e38, 1e-40], np.float32)
    b = sh.from_bf16(sh.to_bf16(x))
    assert b[0] == 1 and b[1] == 1 and b[2] == np.float32(1.0 + 2 ** -6)
    assert np.array_equal(sh.to_bf16(b), sh.to_bf16(x))


# ---- registry and loader (a record-only device: everything up to the first launch) ----------------------------------------------------------
LOADER = r"""
import sys
import crabml_amd as ca
dev = ca.HipTensorDevice(mode="dry")
try:
    ca.load_model(sys.argv[1], dev, seq_len=64)
except ca.CrabmlError as e:
    print(e)
"""


def load_error(path):
    env = dict(os.environ, CRABML_HIP_TEST_HOOKS="1", PYTHONPATH=ROOT)
    p = subprocess.run([sys.executable, "-c", LOADER, path], capture_output=True, text=True, env=env, timeout=60)
    assert p.returncode == 0, p.stderr
    return p.stdout


def write(folder, config=CONFIG, edit=None):
    bits = sh.random_tensors(CONFIG, 1)
    if edit:
        edit(bits)
    return sh.write_model(config, bits, str(folder))


def changed(*path, value):
    c = json.loads(json.dumps(CONFIG))
    at = c
    for p in path[:-1]:
        at = at[p]
    if value is KeyError:
        del at[path[-1]]
    else:
        at[path[-1]] = value
    return c


def test_registry_knows_both_kinds_of_models(ca, tmp_path):
    assert {"Nilivik", "Bifazen", "llama"} <= set(ca.known_architectures())
    assert ca.model_architecture(write(tmp_path / "m")) == "Nilivik"
    assert ca.model_architecture(os.path.join(ROOT, "tests", "golden", "tinyllamas-stories-260k-f32.gguf")) == "llama"
    with pytest.raises(ca.CrabmlError):
        ca.model_architecture(str(tmp_path / "nothing"))


def test_a_good_folder_gets_as_far_as_the_device(tmp_path):
    assert "record-only" in load_error(write(tmp_path / "m"))
    c = changed("loop", value=None)
    assert "record-only" in load_error(write(tmp_path / "n", c))


@pytest.mark.parametrize("path,value,says", [
    (("architecture",), "Other", "unsupported architecture Other"),
    (("width",), KeyError, "missing `width`"),
    (("width",), 48, "is [30, 40]"),
    (("vocab",), 30.5, "whole number"),
    (("layers", 0, "type"), "solo", "unknown mixer `solo`"),
    (("layers", 0, "mlp", "kind"), "sparse", "unknown feed-forward `sparse`"),
    (("layers", 0, "mixer", "right", "decay"), [0.5], "one number per head"),
    (("layers", 1, "mixer", "left", "kv_heads"), 2, "the configuration wants"),
    (("layers", 0, "mixer", "left", "mask", "size"), 0, "chunk size"),
    (("loop", "times"), 3, "loop.step"),
])
def test_wrong_configurations_are_named(tmp_path, path, value, says):
    assert says in load_error(write(tmp_path / "m", changed(*path, value=value)))


def test_wrong_tensor_files_are_named(tmp_path):
    assert "failed to find tensor l0.mix.left.sink" in load_error(write(tmp_path / "a", edit=lambda b: b.pop("l0.mix.left.sink")))
    assert "l1.mix.right.o" in load_error(write(tmp_path / "b", edit=lambda b: b.update({"l1.mix.right.o": b["l1.mix.right.o"].T.copy()})))
    d = write(tmp_path / "c")
    st = os.path.join(d, "model.safetensors")
    raw = open(st, "rb").read()
    for cut in (raw[:4], raw[:40], raw[:-10], b"\xff" * 16 + raw[16:]):
        open(st, "wb").write(cut)
        assert "ErrorKind(6)" in load_error(d), len(cut)
    open(os.path.join(d, "config.json"), "w").write('{"architecture": "Nilivik", ')
    assert "json" in load_error(d)


@pytest.mark.parametrize("text", ['{"a": [1, -2.5e3, true, false, null, "x\\u00e9\\n\\"\\ud83d\\ude00"]}', "[]", " 7 ", '{"k": {}}'])
def test_json_reader_takes_what_json_takes(tmp_path, text):
    """through the loader: valid JSON that is no configuration is a model error or a missing field, never a format error"""
    os.makedirs(tmp_path / "m")
    (tmp_path / "m" / "config.json").write_text(text)
    out = load_error(str(tmp_path / "m"))
    assert "ErrorKind(4)" in out, out
