"""CPU: the configuration registry of the layer-list decoders, and the numpy restatement's own consistency."""
import copy
import json

import numpy as np
import pytest

import layered_util as U
from layered_util import LO

SMALL = U.config(48, 50, [U.layer(U.attention(2, 1, 12, 20, 6, 9, 2), U.delta(2, 1, 10, 14, 3), U.moe(24, 6, 2, (3, 2))),
                          U.layer(U.attention(2, 2, 8, 8, 8, 5, 0), U.delta(3, 3, 6, 4, 2), None)])


def test_registry_takes_the_configuration(tk):
    tk.config_check(SMALL)


@pytest.mark.parametrize("path,value,word", [
    (("architecture",), "Nothing", "not registered"), (("width",), 0, "width"), (("norm", "eps"), None, "eps"),
    (("layers", 0, "type"), "serial", "type"), (("layers", 0, "mixer", "left", "heads"), 3.5, "heads"),
    (("layers", 0, "mixer", "left", "kv_heads"), 3, "multiple"), (("layers", 0, "mixer", "left", "rot", "dims"), 5, "odd"),
    (("layers", 0, "mixer", "right", "dim"), 4096, "dim"), (("layers", 0, "mixer", "right_scale"), None, "right_scale"),
    (("layers", 0, "mlp", "kind"), "sparse", "kind"), (("layers", 0, "mlp", "router", "groups", "count"), 4, "groups"),
    (("layers", 0, "mlp", "router", "top"), 5, "top"), (("layers",), [], "layers")])
def test_registry_names_what_it_refuses(tk, path, value, word):
    c = copy.deepcopy(SMALL)
    at = c
    for k in path[:-1]:
        at = at[k]
    at[path[-1]] = value
    with pytest.raises(tk.TkError) as e:
        tk.config_check(c)
    assert word in str(e.value)


def test_registry_reads_absent_and_null_parts(tk):
    c = copy.deepcopy(SMALL)
    del c["layers"][0]["mlp"]["router"]["groups"]
    c["layers"][0]["mixer"]["left"]["mask"] = None
    del c["layers"][1]["mlp"]
    tk.config_check(c)
    with pytest.raises(tk.TkError):
        tk.config_check("{")
    with pytest.raises(tk.TkError):
        tk.config_check(json.dumps([1, 2]))


def test_layered_model_needs_a_device(tk, tmp_path):
    if tk.lib().tk_mi355x_device_count() > 0:
        pytest.skip("a device is there")
    U.write_folder(tmp_path, SMALL, {})
    for make in (lambda: tk.LlmModel(folder=str(tmp_path)), lambda: tk.LlmModel(config=SMALL)):
        with pytest.raises(tk.TkError) as e:
            make()
        assert e.value.code == 5001


# ---- the restatement against other ways of computing the same thing ----

def test_delta_rule_recurrence_against_its_unrolled_form():
    """S_t = sum over s of (prod of decays) k_s u_s^T with u_s from the triangular system: solved directly for one head"""
    rng = np.random.default_rng(1)
    T, dim, vdim = 9, 5, 4
    q, k, v = rng.standard_normal((T, 1, dim)), rng.standard_normal((T, 1, dim)), rng.standard_normal((T, 1, vdim))
    beta, g = rng.uniform(0.1, 0.9, (T, 1)), rng.uniform(0.5, 1.0, (T, 1, dim))
    o = LO.gated_delta_rule(q, k, v, beta, g)[:, 0]
    G = np.cumprod(g[:, 0], axis=0)
    K, Q = k[:, 0] / G, q[:, 0] * G
    A = np.tril((k[:, 0] * G) @ K.T, -1) * beta
    u = np.linalg.solve(np.eye(T) + A, beta * v[:, 0])
    assert np.allclose(o, np.tril(Q @ K.T) @ u)


def test_router_groups_by_hand():
    s = np.array([0.9, 0.1, 0.2, 0.6, 0.55, 0.5, 0.3, 0.8])
    # pairs sum to 1.0, 0.8, 1.05, 1.1: the last group wins although the first holds the best expert
    assert LO.route(s, 2, 4, 1) == [7, 6]
    assert LO.route(s, 3, 4, 2) == [7, 4, 5]
    assert LO.route(s, 2, 1, 1) == [0, 7]


def test_window_edges_by_hand():
    assert [j for j in range(12) if LO.visible(9, j, 4, 2)] == [0, 1, 6, 7, 8, 9]
    assert [j for j in range(4) if LO.visible(2, j, 4, 2)] == [0, 1, 2]


def test_rotation_keeps_lengths_and_depends_on_distance_only():
    rng = np.random.default_rng(2)
    x, y = rng.standard_normal(10), rng.standard_normal(10)
    at = lambda v, p: LO.rotate_half(v[None, None], np.array([float(p)]), 6, 100.0)[0, 0]
    assert np.isclose(np.linalg.norm(at(x, 7)), np.linalg.norm(x))
    assert np.isclose(at(x, 7) @ at(y, 3), at(x, 11) @ at(y, 7))
    assert np.array_equal(at(x, 7)[6:], x[6:])


def test_causal_convolution_by_hand():
    y = LO.causal_conv(np.array([[1.0], [2.0], [3.0]]), np.array([[10.0, 1.0]]))
    assert y[:, 0].tolist() == [1.0, 12.0, 23.0]
