"""CPU side of the Bifazen design: its plain implementation checked against direct loops, and what the loader says about files that are
not right (a record-only device: everything up to the first launch)."""
import json

import numpy as np
import pytest

from crabml_amd import synth_bifazen as sb
from crabml_amd import synth_hybrid as sh
from tests import bifazen_oracle as bo
from tests.test_hybrid_host import load_error

CONFIG = sb.config(40, 30, [sb.latent(2, 8, 4, 12, 20, 5, 24), sb.attention(4, 2, 8, 10, 9, None), sb.attention(2, 2, 6, 10, 4, 16)], streams=3)


@pytest.fixture(scope="module")
def model():
    return {k: sh.from_bf16(v) for k, v in sb.random_tensors(CONFIG, 3).items()}


def test_oracle_is_causal(model):
    t = [3, 1, 4, 1, 5, 9, 2, 6, 5, 3, 5, 8]
    full = bo.forward(CONFIG, model, t)
    for n in (1, 5, 6, 11):
        assert np.allclose(bo.forward(CONFIG, model, t[:n]), full[:n], rtol=0, atol=1e-10)


def test_oracle_window_against_a_loop_over_keys():
    rng = np.random.default_rng(0)
    T, dv, size = 23, 4, 7
    s, v = rng.standard_normal((T, T)), rng.standard_normal((T, dv))
    got = bo.softmax_attention(s, v, bo.window_mask(T, size))
    for i in range(T):
        js = range(max(0, i - size + 1), i + 1)
        w = np.exp([s[i, j] for j in js])
        assert np.allclose(got[i], (w / w.sum()) @ v[list(js)], atol=1e-12)


def test_oracle_rotation_is_a_rotation_of_neighbours_and_sees_differences_only():
    rng = np.random.default_rng(1)
    q, k = rng.standard_normal((1, 1, 10)), rng.standard_normal((1, 1, 10))
    for shift in (1, 30):
        a = (bo.rotate_pairs(q, [7], 100.0, 6) * bo.rotate_pairs(k, [3], 100.0, 6)).sum()
        b = (bo.rotate_pairs(q, [7 + shift], 100.0, 6) * bo.rotate_pairs(k, [3 + shift], 100.0, 6)).sum()
        assert np.isclose(a, b)
    r = bo.rotate_pairs(q, [1], 100.0, 6)
    assert np.allclose(r[..., 6:], q[..., 6:])
    assert np.isclose(r[0, 0, 0], q[0, 0, 0] * np.cos(1) - q[0, 0, 1] * np.sin(1))
    assert np.isclose(r[0, 0, 5], q[0, 0, 5] * np.cos(100 ** (-4 / 6)) + q[0, 0, 4] * np.sin(100 ** (-4 / 6)))


def test_oracle_latent_scores_may_be_taken_in_the_latent(model):
    """q . (W c) = (W^T q) . c, which the decode step relies on"""
    rng = np.random.default_rng(2)
    w = model["l0.mix.uk"].reshape(2, 8, 20).astype(np.float64)
    q, c = rng.standard_normal((2, 8)), rng.standard_normal(20)
    assert np.allclose([q[h] @ (w[h] @ c) for h in range(2)], [(w[h].T @ q[h]) @ c for h in range(2)])


def test_oracle_single_stream_that_keeps_itself_is_a_residual_sum(model):
    xs = np.random.default_rng(3).standard_normal((1, 4, 6))
    w = {"in": np.ones(1), "out": np.ones(1), "mix": np.ones((1, 1))}
    assert np.allclose(bo.hyper_connection(xs, w, "", lambda u: 2 * u)[0], 3 * xs[0])


def test_oracle_mixing_matrix_is_from_to(model):
    xs = np.random.default_rng(4).standard_normal((2, 3, 5))
    w = {"in": np.array([1.0, 0.0]), "out": np.zeros(2), "mix": np.array([[0.0, 1.0], [0.0, 0.0]])}
    got = bo.hyper_connection(xs, w, "", lambda u: u)
    assert np.allclose(got[0], 0) and np.allclose(got[1], xs[0])


def write(folder, config=CONFIG, edit=None):
    bits = sb.random_tensors(CONFIG, 1)
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


def test_a_good_folder_gets_as_far_as_the_device(tmp_path):
    assert "record-only" in load_error(write(tmp_path / "m"))
    assert "record-only" in load_error(write(tmp_path / "n", changed("layers", 1, "mixer", "v_mix", value=KeyError)))


@pytest.mark.parametrize("path,value,says", [
    (("width",), KeyError, "missing `width`"),
    (("width",), 48, "is [30, 40]"),
    (("streams",), KeyError, "missing `streams`"),
    (("streams",), 0, "`streams`"),
    (("streams",), 4, "the configuration wants"),
    (("layers", 0, "type"), "solo", "unknown mixer `solo`"),
    (("layers", 0, "mlp", "kind"), "sparse", "unknown feed-forward `sparse`"),
    (("layers", 0, "mixer", "rot", "dims"), 2, "rot_dim"),
    (("layers", 0, "mixer", "kv_rank"), 24, "l0.mix.dkv"),
    (("layers", 0, "mixer", "mask", "size"), 0, "window size"),
    (("layers", 1, "mixer", "kv_heads"), 4, "the configuration wants"),
    (("layers", 1, "mixer", "v_mix"), 1, "true or false"),
    (("norm", "eps"), KeyError, "missing `eps`"),
])
def test_wrong_configurations_are_named(tmp_path, path, value, says):
    assert says in load_error(write(tmp_path / "m", changed(*path, value=value)))


def test_wrong_tensor_files_are_named(tmp_path):
    for name in ("l0.hc1.mix", "l0.mix.dkv.norm", "l1.mix.q.b", "l2.mix.vmix", "final.norm"):
        assert "failed to find tensor " + name in load_error(write(tmp_path / name, edit=lambda b: b.pop(name)))
    assert "l0.mix.o" in load_error(write(tmp_path / "o", edit=lambda b: b.update({"l0.mix.o": b["l0.mix.o"].T.copy()})))
