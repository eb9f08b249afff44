"""Zedenex model folders on the host, and checks of the plain evaluation that the device tests compare against."""
import copy
import importlib
import json
import os

import numpy as np
import pytest

import block_builder as bb
import zedenex_builder as zb
import zedenex_oracle as zo


@pytest.fixture(scope="module")
def hostlib():
    return importlib.import_module("llama-vulkan_amd.hostlib")


def _open(hostlib, folder):
    c = hostlib.LlavaContext()
    ok, err = c.open_model_file(folder), c.error()
    c.close()
    return ok, err


def test_folder_opens_and_refusals_name_their_reason(hostlib, tmp_path):
    cfg = zb.config(loop=(1, 3, 2))
    good = str(tmp_path / "good")
    W = bb.write_folder(good, cfg, W=zb.weights(cfg, 1))
    assert W["l0.norm1.alpha"].shape == ()
    assert _open(hostlib, good) == (True, "")

    def opened(change, name):
        c = copy.deepcopy(cfg)
        change(c)
        p = str(tmp_path / name)
        os.mkdir(p)
        os.symlink(os.path.join(good, "model.safetensors"), os.path.join(p, "model.safetensors"))
        with open(os.path.join(p, "config.json"), "w") as f:
            json.dump(c, f)
        return _open(hostlib, p)
    for i, change in enumerate((lambda c: c.pop("loop"), lambda c: c.update(loop=None), lambda c: c["embedding"].pop("bigram"), lambda c: c["layers"][0].pop("mlp"),
                                lambda c: c["embedding"]["bigram"].update(mul_prev=10 ** 12))):
        assert opened(change, f"fine{i}") == (True, "")
    for i, (word, change) in enumerate((("type", lambda c: c["layers"][1].update(type="windowed")), ("feed-forward", lambda c: c["layers"][0]["mlp"].update(kind="moe")),
                                        ("kv_rank", lambda c: c["layers"][0]["mixer"].pop("kv_rank")), ("streams", lambda c: c.update(streams=0)),
                                        ("loop", lambda c: c["loop"].update(stop=5)), ("loop", lambda c: c["loop"].update(times=0)),
                                        ("buckets", lambda c: c["embedding"]["bigram"].update(buckets=0)), ("whole number", lambda c: c["layers"][1]["mixer"].update(state=2.5)))):
        ok, err = opened(change, f"bad{i}")
        assert not ok and word in err, (word, err)


# ---- the plain evaluation ----------------------------------------------------------------------------------------------
def test_bigram_rows():
    W = {"embed": np.zeros((9, 1)), "bigram": np.arange(6.0)[:, None]}
    c = {"scale": 3.0, "bigram": {"buckets": 5, "mul_prev": 2, "mul_cur": 7}}
    assert zo.embedding([4, 1, 8], W, c)[:, 0].tolist() == [5.0, (4 * 2 + 7) % 5, (1 * 2 + 8 * 7) % 5]
    W["embed"][4] = 2.0
    assert zo.embedding([4], W, {"scale": 3.0})[0, 0] == 6.0


def test_streams_from_to():
    x = np.array([1.0, 10.0])[:, None, None]
    mix = np.array([[1.0, 2.0], [3.0, 4.0]])              # [from, to]
    new = zo.spread_streams(x, mix, np.array([0.5, -1.0]), np.array([[100.0]]))
    assert new[:, 0, 0].tolist() == [1 + 30 + 50, 2 + 40 - 100]
    assert zo.gather_streams(x, np.array([2.0, 0.1]))[0, 0] == 3.0


def test_run_order():
    cfg = {"layers": [0] * 5, "loop": {"start": 1, "stop": 3, "times": 3}}
    assert zo.run_order(cfg) == [0, 1, 2, 1, 2, 1, 2, 3, 4]
    assert zo.run_order({"layers": [0] * 2}) == [0, 1]


def test_state_space_closed_form():
    # no decay (dt tiny against A), a step size of one: the state is the sum of outer products; D passes x
    n, rng = 5, np.random.default_rng(0)
    x, B, C = rng.standard_normal((n, 1, 2)), rng.standard_normal((n, 1, 3)), rng.standard_normal((n, 1, 3))
    y = zo.state_space(x, B, C, np.ones((n, 1)), np.array([-40.0]), np.array([0.0]))
    want = [sum((C[t, 0] @ B[s, 0]) * x[s, 0] for s in range(t + 1)) for t in range(n)]
    assert np.allclose(y[:, 0], want)
    # a rate of log 2 per token halves what is there before the write
    y = zo.state_space(np.ones((3, 1, 1)), np.ones((3, 1, 1)), np.ones((3, 1, 1)), np.ones((3, 1)), np.log([np.log(2.0)]), np.array([10.0]))
    assert np.allclose(y[:, 0, 0], [11.0, 11.5, 11.75])


def test_convolution_bias_and_order():
    y = zo.biased_causal_conv(np.array([[0.0], [1.0], [0.0], [0.0]]), np.array([[5.0, 7.0]]), np.array([0.5]))
    assert np.allclose(y[:, 0], zo.silu(np.array([0.5, 7.5, 5.5, 0.5])))


def test_latent_attention_is_ordinary_attention_over_expanded_keys():
    """one head, no rotation: softmax over (W_uk c) with values W_uv c; and a score depends on the distance only"""
    rng = np.random.default_rng(3)
    c = zb.latent(heads=1, dim=4, rot_dim=2, vdim=3, q_rank=5, kv_rank=6)
    W = {k: rng.standard_normal(s) for k, s in (("dq", (5, 8)), ("uq", (6, 5)), ("dkv", (8, 8)), ("uk", (4, 6)), ("uv", (3, 6)), ("o", (8, 3)), ("dq.norm", 5), ("dkv.norm", 6))}
    W["uq"][4:] = 0
    h = rng.standard_normal((7, 8))
    lat = zo.rms_norm(h @ W["dkv"][:6].T, W["dkv.norm"], 1e-5)
    q = zo.rms_norm(h @ W["dq"].T, W["dq.norm"], 1e-5) @ W["uq"][:4].T
    s = np.where(np.tril(np.ones((7, 7), bool)), q @ (lat @ W["uk"].T).T * c["scale"], -np.inf)
    e = np.exp(s - s.max(1, keepdims=True))
    want = (e / e.sum(1, keepdims=True)) @ (lat @ W["uv"].T) @ W["o"].T
    assert np.allclose(zo.latent_attention(h, W, "", c, 1e-5), want)


def test_grouped_norm_and_tanh():
    x = np.array([[3.0, 4.0, 0.0, 2.0]])
    y = zo.grouped_rms_norm(x, 2, np.array([1.0, 1.0, 1.0, 10.0]), 0.0)
    assert np.allclose(y, [[3 / 12.5 ** 0.5, 4 / 12.5 ** 0.5, 0, 10 * 2 ** 0.5]])
    assert np.allclose(zo.dynamic_tanh(np.array([0.5]), 2.0, 3.0, 4.0), 3 * np.tanh(1.0) + 4)
