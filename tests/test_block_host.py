"""Block models on the host: reading a model folder, token ids as text, and checks of the plain evaluation that the device
tests compare against."""
import copy
import importlib
import json
import os

import numpy as np
import pytest

import block_builder as bb
import block_oracle as bo


@pytest.fixture(scope="module")
def hostlib():
    return importlib.import_module("llama-vulkan_amd.hostlib")


def _open(hostlib, folder):
    c = hostlib.LlavaContext()
    ok = c.open_model_file(folder)
    err = c.error()
    c.close()
    return ok, err


def test_folder_opens_and_refusals_name_their_reason(hostlib, tmp_path):
    cfg = bb.config()
    good = str(tmp_path / "good")
    bb.write_folder(good, cfg, seed=1)
    assert _open(hostlib, good) == (True, "")

    def broken(change, name):
        c = copy.deepcopy(cfg)
        change(c)
        p = str(tmp_path / name)
        bb.write_folder(p, cfg, seed=1)
        with open(os.path.join(p, "config.json"), "w") as f:
            json.dump(c, f)
        ok, err = _open(hostlib, p)
        assert not ok
        return err
    assert "Othersun" in broken(lambda c: c.update(architecture="Othersun"), "arch")
    assert "recurrent" in broken(lambda c: c["layers"][1].update(type="recurrent"), "type")
    assert "dense" in broken(lambda c: c["layers"][0]["mlp"].update(kind="dense"), "kind")
    assert "heads" in broken(lambda c: c["layers"][0]["mixer"]["left"].pop("heads"), "missing")
    assert "whole number" in broken(lambda c: c["layers"][0]["mixer"]["right"].update(conv=2.5), "fraction")
    empty = str(tmp_path / "empty")
    os.mkdir(empty)
    assert not _open(hostlib, empty)[0]
    os.remove(os.path.join(good, "model.safetensors"))
    assert not _open(hostlib, good)[0]


# ---- the plain evaluation ----------------------------------------------------------------------------------------------
def test_rotation_depends_on_distance_only():
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((1, 1, 10)), rng.standard_normal((1, 1, 10))

    def score(i, j):
        return float(bo.rotate(q, np.array([float(i)]), 6, 50.0)[0, 0] @ bo.rotate(k, np.array([float(j)]), 6, 50.0)[0, 0])
    assert abs(score(9, 4) - score(25, 20)) < 1e-12
    assert abs(score(9, 4) - score(9, 5)) > 1e-3
    x = rng.standard_normal((3, 2, 10))
    assert np.array_equal(bo.rotate(x, np.arange(3.0), 6, 50.0)[:, :, 6:], x[:, :, 6:])
    # a quarter turn takes (u, v) to (-v, u)
    assert np.allclose(bo.rotate(np.array([[[1.0, 0.0]]]), np.array([np.pi / 2]), 2, 7.0), [[[0.0, 1.0]]])


def test_chunk_visibility_and_sink():
    m = bo.visible(7, 3)
    assert [int(r.sum()) for r in m] == [1, 2, 3, 1, 2, 3, 1]
    assert m[4, 3] and not m[3, 2] and not m[3, 4]
    assert bo.visible(5, 0).sum() == 15
    w = bo.sink_softmax(np.zeros((1, 4)), np.ones((1, 4), bool), np.log(4.0))
    assert np.allclose(w, 1 / 8)
    assert np.allclose(bo.sink_softmax(np.array([[800.0, 0.0]]), np.ones((1, 2), bool), 800.0), [[0.5, 0.0]])


def test_convolution_of_an_impulse_plays_the_taps_backwards():
    w = np.array([[1.0, 2.0, 3.0]])
    x = np.zeros((5, 1))
    x[1] = 1.0
    assert np.allclose(bo.causal_conv(x, w)[:, 0], bo.silu(np.array([0.0, 3.0, 2.0, 1.0, 0.0])))


def test_delta_recurrence_closed_forms():
    # decay 1, step 1, orthonormal keys: the state is an exact store, and writing a key again replaces its value
    eye = np.eye(3)
    k = np.stack([eye[0], eye[1], eye[0]])[:, None]
    v = np.array([[1.0, 2.0], [3.0, 4.0], [5.0, 6.0]])[:, None]
    one = np.ones((3, 1, 3))
    q = np.stack([eye[0], eye[0] + eye[1], eye[0] + eye[1]])[:, None]
    o = bo.delta_recurrence(q, k, v, np.ones((3, 1)), one)
    assert np.allclose(o[:, 0], [[1, 2], [4, 6], [8, 10]])
    # decay acts on the key's row before the write: channel 0 halves at the second token
    g = one.copy()
    g[1, 0, 0] = 0.5
    o = bo.delta_recurrence(q, k, v, np.ones((3, 1)), g)
    assert np.allclose(o[1, 0], [0.5 + 3, 1 + 4])


def test_mixture_weights_its_experts_inputs():
    W = {"router": np.array([[2.0, 0.0], [1.0, 0.0], [-1.0, 0.0]])}
    for e in range(3):
        W[f"e{e}.gate"], W[f"e{e}.up"], W[f"e{e}.down"] = np.array([[1.0, 0.0]]), np.array([[0.0, 1.0]]), np.array([[1.0], [0.0]])
    h = np.array([[1.0, 3.0]])
    want = sum(bo.silu(s) * (s * 3.0) for s in (bo.sigmoid(2.0), bo.sigmoid(1.0)))
    assert np.allclose(bo.mixture(h, W, "", 2)[0], [want, 0.0])
    assert bo.choose_experts(np.array([1.0, 2.0, 2.0]), 2).tolist() == [1, 2]
