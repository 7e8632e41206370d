"""CPU: Kaparax in the configuration registry, and the restatement's mechanisms against other derivations."""
import copy

import numpy as np
import pytest

import layered_util as U
from layered_util import LO

SMALL = U.kaparax(40, 50, [U.serial(U.retention(3, 10, 14, 6, [0.5, 0.9, 1.0])),
                           U.serial(U.chunked(4, 2, 12, 20, 6, 9, 3, 8.0), (24, 2.5)),
                           U.serial(U.retention(3, 10, 14, 6, [0.5, 0.9, 1.0]), None, 0),
                           U.serial(U.chunked(4, 2, 12, 20, 6, 9, 3, 8.0), (24, 2.5), 1)], scale=3.5)


def at_path(path, value):
    c = copy.deepcopy(SMALL)
    at = c
    for k in path[:-1]:
        at = at[k]
    at[path[-1]] = value
    return c


def test_registry_takes_the_configuration(tk):
    tk.config_check(SMALL)


@pytest.mark.parametrize("path,value", [(("layers", 1, "mixer", "mask"), None), (("layers", 3, "weights_of"), None), (("layers", 0, "mlp"), {"kind": "dense", "ff": 7, "limit": 1}),
                                        (("layers", 1, "mixer", "softcap"), None), (("layers", 0, "mixer", "rot", "dims"), 0), (("layers", 0, "mixer", "decay"), [0.0, 1.0, 0.3])])
def test_registry_takes_variants(tk, path, value):
    c = at_path(path, value)
    if path[0] == "layers" and path[1] == 0 and path[2] == "mlp":
        c["layers"][2]["mlp"] = value
    tk.config_check(c)


@pytest.mark.parametrize("path,value,word", [
    (("embedding",), None, "embedding"), (("embedding", "scale"), "x", "scale"), (("layers", 0, "type"), "parallel", "type"),
    (("layers", 0, "mixer", "decay"), [0.5, 0.5], "decay"), (("layers", 0, "mixer", "decay"), [0.5, 0.5, 1.5], "decay"), (("layers", 0, "mixer", "dim"), 4096, "dim"),
    (("layers", 0, "mixer", "rot", "dims"), 5, "odd"), (("layers", 1, "mixer", "kv_heads"), 3, "multiple"), (("layers", 1, "mixer", "mask", "size"), 0, "size"),
    (("layers", 1, "mixer", "softcap"), -1.0, "softcap"), (("layers", 1, "mixer", "conv"), 99, "conv"), (("layers", 1, "mlp", "limit"), None, "limit"),
    (("layers", 1, "mlp", "kind"), "moe", "expert"), (("layers", 2, "weights_of"), 1, "other sizes"), (("layers", 2, "weights_of"), 9, "weights_of"),
    (("layers", 2, "weights_of"), 2, "itself"), (("norm", "eps"), None, "eps"), (("layers", 3, "mixer"), None, "mixer")])
def test_registry_names_what_it_refuses(tk, path, value, word):
    with pytest.raises(tk.TkError) as e:
        tk.config_check(at_path(path, value))
    assert word in str(e.value)


def test_layers_may_borrow_from_borrowers(tk):
    tk.config_check(at_path(("layers", 2, "weights_of"), 0))
    c = copy.deepcopy(SMALL)
    c["layers"].append(U.serial(c["layers"][0]["mixer"], None, 2))
    tk.config_check(c)
    w = U.random_weights(c, 3)
    assert not any(k.startswith(("l2.", "l3.", "l4.")) for k in w)
    direct = copy.deepcopy(c)
    direct["layers"][4]["weights_of"] = 0
    assert np.array_equal(LO.forward(c, w, [1, 2, 3])[0], LO.forward(direct, w, [1, 2, 3])[0])


# ---- the restatement against other ways of computing the same thing ----

def test_retention_recurrence_against_its_parallel_form():
    rng = np.random.default_rng(1)
    q, k, v = rng.standard_normal((9, 2, 5)), rng.standard_normal((9, 2, 5)), rng.standard_normal((9, 2, 4))
    decay = [0.8, 1.0]
    o = LO.retention(q, k, v, decay)
    t = np.arange(9)
    for h in range(2):
        fade = np.where(t[:, None] >= t, np.power(decay[h], np.maximum(t[:, None] - t, 0)), 0.0)
        assert np.allclose(o[:, h], (q[:, h] @ k[:, h].T * fade) @ v[:, h])


def test_chunks_by_hand():
    assert [j for j in range(12) if LO.same_chunk(9, j, 4)] == [8, 9]
    assert [j for j in range(12) if LO.same_chunk(7, j, 4)] == [4, 5, 6, 7]
    assert [j for j in range(12) if LO.same_chunk(8, j, 4)] == [8]
    assert [j for j in range(4) if LO.same_chunk(2, j, None)] == [0, 1, 2]


def test_attention_of_one_chunk_against_matrices():
    rng = np.random.default_rng(5)
    q, k, v = rng.standard_normal((6, 4, 3)), rng.standard_normal((6, 2, 3)), rng.standard_normal((6, 2, 7))
    o = LO.chunked_attention(q, k, v, 0.7, 100, 1.5)
    s = 1.5 * np.tanh(0.7 * q[:, 3] @ k[:, 1].T / 1.5)
    e = np.tril(np.exp(s))
    assert np.allclose(o[:, 3], e / e.sum(1, keepdims=True) @ v[:, 1])


def test_clamped_gate_by_hand():
    w = {"gate": np.array([[1.0]]), "up": np.array([[1.0]]), "down": np.array([[2.0]])}
    f = lambda z: LO.clamped_glu(w, "", np.array([[z]]), 3.0)[0, 0] / 2.0
    sig = lambda z: 1.0 / (1.0 + np.exp(-1.702 * z))
    assert np.isclose(f(1.0), 1.0 * sig(1.0) * 2.0)
    assert np.isclose(f(50.0), 3.0 * sig(3.0) * 4.0)
    assert np.isclose(f(-2.0), -2.0 * sig(-2.0) * -1.0)
    assert np.isclose(f(-5.0), -5.0 * sig(-5.0) * -2.0)  # the gate is not cut below


def test_layer_norm_by_hand():
    x = LO.layer_norm(np.array([[1.0, 3.0]]), np.array([2.0, 2.0]), np.array([0.5, -0.5]), 0.0)
    assert np.allclose(x, [[-1.5, 1.5]])
    assert LO.layer_norm(np.array([[4.0, 4.0]]), np.ones(2), np.zeros(2), 1e-5).tolist() == [[0.0, 0.0]]
