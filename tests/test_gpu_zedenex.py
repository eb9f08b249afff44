"""Zedenex models on the device, and their mechanisms in other combinations, against the plain evaluation of
tests/zedenex_oracle.py: every mechanism alone, prompts, decoding, portions, keys and states that stand out, sessions that are
used again, and generation through the host classes.

Sizes are odd on purpose (no power of two, heads that do not fill a tile, ranks that are no multiple of anything).  In 32-bit the
device agrees to 32-bit rounding; in bfloat16 to the rounding of matrix product operands."""
import importlib
import json
import os
import subprocess

import numpy as np
import pytest

import block_builder as bb
import server_client as sc
import zedenex_builder as zb
import zedenex_oracle as zo
from block_device import Device, rel, tokens_for

pytestmark = pytest.mark.gpu
F32, BF16 = 0, 30
TOL = {F32: 3e-5, BF16: 5e-2}


@pytest.fixture(scope="module")
def hostlib():
    return importlib.import_module("llama-vulkan_amd.hostlib")


def device(lva, ctx, cfg, W, compute, backlog=512):
    return Device(lva, zb.upload(ctx, cfg, W, compute), backlog)


def check_model(lva, ctx, cfg, W, n, compute=F32, cuts=((1000,), (1,)), seed=0, tol=None, toks=None):
    """residual behind every sublayer and logits, for prompts cut as given"""
    toks = tokens_for(cfg, n, seed) if toks is None else toks
    want, mid, out = zo.forward(toks, bb.as_float(W), cfg)
    tol = tol or TOL[compute]
    with device(lva, ctx, cfg, W, compute) as d:
        d.sess.trace_enable(True)
        for c in cuts:
            got = d.run(toks, c)
            assert rel(got, want) < tol, c
            last = d.sess.trace_all(0, lva.TRACE_OUT).shape[0]        # rows of the last portion
            for i in range(len(out)):
                assert rel(d.sess.trace_all(i, lva.TRACE_POST_ATTN), mid[i][-last:]) < tol, ("mixer", i, c)
                assert rel(d.sess.trace_all(i, lva.TRACE_OUT), out[i][-last:]) < tol, ("layer", i, c)
        d.sess.trace_enable(False)
        for c in cuts:
            assert rel(d.run(toks, c), want) < tol, ("untraced", c)
    return want


# ---- each mechanism alone ------------------------------------------------------------------------------------------------
LATENT = [
    dict(heads=3, dim=12, rot_dim=6, vdim=10, q_rank=20, kv_rank=18),
    dict(heads=1, dim=40, rot_dim=2, vdim=70, q_rank=7, kv_rank=5),              # values wider than keys, one pair turns
    dict(heads=17, dim=8, rot_dim=8, vdim=9, q_rank=64, kv_rank=64),             # one head more than a tile
    dict(heads=5, dim=100, rot_dim=70, vdim=65, q_rank=130, kv_rank=200),        # padded key size 192
    dict(heads=2, dim=190, rot_dim=64, vdim=33, q_rank=65, kv_rank=72),          # padded key size 256
    dict(heads=33, dim=33, rot_dim=32, vdim=64, q_rank=48, kv_rank=100),         # odd unrotated part
    dict(heads=2, dim=48, rot_dim=16, vdim=128, q_rank=40, kv_rank=600, scale=0.3),   # a wide latent: two pieces a wave
    dict(heads=4, dim=256, rot_dim=0, vdim=256, q_rank=33, kv_rank=16),          # nothing turns
    dict(heads=220, dim=60, rot_dim=8, vdim=9, q_rank=16, kv_rank=24),           # many heads
]


@pytest.mark.parametrize("compute", [F32, BF16])
@pytest.mark.parametrize("k", range(len(LATENT)))
def test_latent_attention_alone(lva, ctx, k, compute):
    cfg = zb.config(width=50, streams=1 + k % 3, layers=[zb.layer(zb.latent(**LATENT[k]), 0)])
    W = zb.weights(cfg, seed=10 + k, sinks=k != 2)
    check_model(lva, ctx, cfg, W, 150, compute, cuts=((1000,), (1,), (37, 2, 16, 64, 3)))


SSM = [
    dict(heads=6, groups=3, state=20, vdim=7, conv=3, norm_groups=2),
    dict(heads=4, groups=4, state=64, vdim=33, conv=1, norm_groups=1),           # no convolution memory, a norm over everything
    dict(heads=3, groups=1, state=70, vdim=16, conv=4, norm_groups=6),           # norm parts that are not heads
    dict(heads=2, groups=2, state=130, vdim=40, conv=6, norm_groups=16),         # more norm parts than waves
    dict(heads=1, groups=1, state=256, vdim=9, conv=2, norm_groups=9),           # norm parts of one entry
    dict(heads=12, groups=2, state=5, vdim=64, conv=5, norm_groups=3),
]


@pytest.mark.parametrize("compute", [F32, BF16])
@pytest.mark.parametrize("k", range(len(SSM)))
def test_state_space_alone(lva, ctx, k, compute):
    cfg = zb.config(width=44, streams=1 + k % 4, layers=[zb.layer(zb.ssm(**SSM[k]), 0)])
    W = zb.weights(cfg, seed=20 + k)
    check_model(lva, ctx, cfg, W, 150, compute, cuts=((1000,), (1,), (37, 2, 16, 31, 3)))


@pytest.mark.parametrize("compute", [F32, BF16])
@pytest.mark.parametrize("ff,width", [(28, 40), (1, 70), (100, 33), (300, 130), (16500, 48)])
def test_dense_feed_forward_alone(lva, ctx, ff, width, compute):
    cfg = zb.config(width=width, layers=[zb.layer(ff=ff)])
    W = zb.weights(cfg, seed=30 + ff)
    W["l0.mix.o"][:] = 0                      # the mixer adds nothing
    check_model(lva, ctx, cfg, W, 70, compute, cuts=((1000,), (1,), (16, 5)))


@pytest.mark.parametrize("compute", [F32, BF16])
@pytest.mark.parametrize("streams", [1, 2, 3, 4, 5, 8])
def test_streams(lva, ctx, streams, compute):
    cfg = zb.config(width=36, streams=streams)
    W = zb.weights(cfg, seed=400 + streams)
    want = check_model(lva, ctx, cfg, W, 60, compute, cuts=((1000,), (1,), (17, 2)))
    if streams > 1:                           # a mix matrix the other way round would show
        F = bb.as_float(W)
        for k in F:
            if k.endswith(".mix") and ".hc" in k:
                F[k] = F[k].T
        assert rel(zo.forward(tokens_for(cfg, 60, 0), F, cfg)[0], want) > 0.05


@pytest.mark.parametrize("bigram", [(31, 7, 3), (1, 5, 9), (1009, 4001, 70001), (64, 0, 1), None])
def test_embedding_remembers_the_previous_token(lva, ctx, bigram):
    """mixers and feed-forwards add nothing: the logits are the embedding's doing.  Portions of even and odd sizes, and single
    tokens between them, hand the previous token on"""
    cfg = zb.config(vocab=70, width=40, streams=2, layers=[zb.layer(), zb.layer(zb.ssm(), 0)], bigram=bigram, scale=3.25)
    W = zb.weights(cfg, 7)
    for k in W:
        if k.endswith("mix.o") or k.endswith("mlp.down"):
            W[k][:] = 0
    check_model(lva, ctx, cfg, W, 120, F32, cuts=((1000,), (1,), (2,), (3,), (16, 1, 17, 1, 1, 18, 2), (20,)), tol=1e-5)
    if bigram and bigram[1]:
        toks, F = tokens_for(cfg, 120, 0), bb.as_float(W)
        want = zo.forward(toks, F, cfg)[0]
        assert rel(zo.forward(toks[1:], F, cfg)[0][:1], want[1:2]) > 0.05 or bigram[0] == 1      # the second token as a first one


# ---- the mechanisms otherwise put together ---------------------------------------------------------------------------------
def with_branches(cfg, i, W, seed, experts=0):
    """layer i becomes attention and delta rule side by side, with a mixture behind them if `experts`"""
    l = bb.layer(experts=experts, top=max(1, experts))
    cfg["layers"][i] = l
    for k in [k for k in W if k.startswith(f"l{i}.mix") or k.startswith(f"l{i}.mlp")]:
        del W[k]
    other = bb.weights({"vocab": 3, "width": cfg["width"], "layers": [l]}, seed)
    for k, v in other.items():
        if k.startswith("l0.mix") or k.startswith("l0.mlp"):
            W[f"l{i}." + k[3:]] = v
    return cfg, W


@pytest.mark.parametrize("compute", [F32, BF16])
@pytest.mark.parametrize("tanh,streams,tied,scale", [(False, 3, True, 2.0), (False, 0, False, 0.0), (True, 2, False, 1.5)])
def test_other_designs(lva, ctx, tanh, streams, tied, scale, compute):
    """RMS norms on streams, a plain residual with norms on both sides, an output matrix of its own, SiLU, layers of attention and
    delta rule with a mixture among the others"""
    cfg = zb.config(streams=streams, scale=scale, bigram=None, layers=[zb.layer(), zb.layer(ff=30), zb.layer(zb.ssm(), 40)], loop=(0, 2, 2))
    W = zb.weights(cfg, 50 + streams, tanh=tanh, tied=tied)
    cfg["layers"][2]["mlp"]["act"] = "silu"
    if not scale:
        cfg["embedding"]["scale"] = 1.0
    with_branches(cfg, 1, W, 3, experts=4)
    n = 40
    want, mid, out = zo.forward(tokens_for(cfg, n, 1), bb.as_float(W), cfg)
    if not scale:
        cfg["embedding"]["scale"] = 0.0       # stands for 1
    tol = {F32: 2e-4, BF16: 0.15}[compute]      # sums of streams can be small, which an RMS norm blows up
    with device(lva, ctx, cfg, W, compute) as d:
        toks = tokens_for(cfg, n, 1)
        for c in ((1000,), (1,), (18, 3)):
            assert rel(d.run(toks, c), want) < tol, c
        assert len(out) == 5
        d.sess.trace_enable(True)
        d.run(toks, (1000,))
        for i in range(5):
            assert rel(d.sess.trace_all(i, lva.TRACE_POST_ATTN), mid[i]) < tol, i
            assert rel(d.sess.trace_all(i, lva.TRACE_OUT), out[i]) < tol, i
        d.sess.trace_enable(False)
        # the last row's logits alone, behind a pending mixture or feed-forward
        d.sess.keep_all_logits(False)
        for m in (n, 1):
            d.sess.begin(toks[:m], 0)
            assert rel(d.sess.logits()[None], want[m - 1:m]) < tol


def test_a_mixture_at_the_end(lva, ctx):
    """several vectors per token wait for the head"""
    cfg = zb.config(streams=2, bigram=None, layers=[zb.layer(), zb.layer(ff=30)])
    W = zb.weights(cfg, 55)
    with_branches(cfg, 1, W, 4, experts=3)
    toks = tokens_for(cfg, 30, 1)
    want = zo.forward(toks, bb.as_float(W), cfg)[0]
    with device(lva, ctx, cfg, W, F32) as d:
        assert rel(d.run(toks, (1000,)), want) < 2e-4
        d.sess.keep_all_logits(False)
        d.sess.begin(toks, 0)
        assert rel(d.sess.logits()[None], want[-1:]) < 2e-4


# ---- whole models --------------------------------------------------------------------------------------------------------
def deep(loop=(1, 4, 3), vocab=67, width=52):
    return zb.config(vocab=vocab, width=width, streams=2, loop=loop, bigram=(97, 13, 29), layers=[
        zb.layer(zb.ssm(heads=3, groups=3, state=12, vdim=20, conv=4, norm_groups=5), 40),
        zb.layer(zb.latent(heads=5, dim=24, rot_dim=8, vdim=16, q_rank=30, kv_rank=26), 0),
        zb.layer(zb.ssm(heads=8, groups=2, state=33, vdim=6, conv=2, norm_groups=1), 0),
        zb.layer(zb.latent(heads=2, dim=10, rot_dim=12, vdim=40, q_rank=50, kv_rank=40, base=3e4, scale=0.4), 33),
        zb.layer(zb.ssm(heads=1, groups=1, state=16, vdim=24, conv=3, norm_groups=2), 0)])


PORTIONS = [(1000,), (2,), (16, 2, 2, 33, 16, 50, 3), (49, 1, 1, 20, 2), (7,), (130, 2), (17,)]


@pytest.mark.parametrize("compute", [F32, BF16])
def test_portions_and_decoding_agree(lva, ctx, compute):
    cfg = deep()
    check_model(lva, ctx, cfg, zb.weights(cfg, 41), 190, compute, cuts=PORTIONS, tol={F32: 1e-4, BF16: 8e-2}[compute])


@pytest.mark.parametrize("loop", [None, (0, 5, 2), (2, 3, 4), (4, 5, 2), (0, 1, 1), (2, 2, 3)])
def test_loops(lva, ctx, loop):
    """a pass has its own cache and state: shared ones would show"""
    cfg = deep(loop)
    W = zb.weights(cfg, 42)
    want = check_model(lva, ctx, cfg, W, 60, F32, cuts=((1000,), (1,), (20, 3)), tol=1e-4)
    if loop and loop[2] > 1 and loop[1] > loop[0]:
        assert rel(zo.forward(tokens_for(cfg, 60, 0), bb.as_float(W), {**cfg, "loop": None})[0], want) > 0.05


@pytest.mark.parametrize("n", [1, 2, 3, 4, 15, 16, 17, 31, 32, 33])
def test_first_tokens(lva, ctx, n):
    """shorter than a convolution, shorter than a batch, a block of keys and just around one"""
    cfg = deep()
    check_model(lva, ctx, cfg, zb.weights(cfg, 43), n, F32, cuts=((n,), (1,)), tol=1e-4)


def test_a_prompt_longer_than_a_batch(lva, ctx):
    """2150 tokens: two batches inside one step, the wide forms of matrix product and attention tiles; then decoding with more
    blocks of keys than there are key ranges"""
    cfg = zb.config(vocab=4099, width=72, layers=[zb.layer(zb.latent(heads=32, dim=128, rot_dim=10, vdim=128, q_rank=40, kv_rank=30), 2100), zb.layer(zb.ssm(), 0)], bigram=(97, 13, 29))
    W = zb.weights(cfg, 48)
    toks = tokens_for(cfg, 2150, 4)
    want = zo.forward(toks, bb.as_float(W), cfg)[0]
    for compute in (BF16, F32):
        with device(lva, ctx, cfg, W, compute, backlog=2200) as d:
            assert rel(d.run(toks, (2150,)), want) < TOL[compute]
            d.step(toks[:2090], 0)
            assert rel(d.run(toks, (2049, 81, 1)), want) < TOL[compute]


@pytest.mark.parametrize("compute", [F32, BF16])
def test_more_key_blocks_than_ranges(lva, ctx, compute):
    """many heads leave few key ranges a head: several blocks each, the last range with fewer or none"""
    cfg = zb.config(width=40, streams=1, layers=[zb.layer(zb.latent(heads=250, dim=4, rot_dim=2, vdim=3, q_rank=16, kv_rank=12), 0)])
    W = zb.weights(cfg, 49)
    toks = tokens_for(cfg, 1060, 4)
    want = zo.forward(toks, bb.as_float(W), cfg)[0]
    with device(lva, ctx, cfg, W, compute, backlog=1100) as d:
        for first in (500, 700, 1020):
            assert rel(d.run(toks[:first + 40], (first, 1)), want[:first + 40]) < TOL[compute], first


def test_long_decoding_follows_the_prompt_form(lva, ctx):
    """420 tokens decoded one by one through graph replays, the cache growing under them"""
    cfg = deep()
    W = zb.weights(cfg, 44)
    toks = tokens_for(cfg, 440, 5)
    want = zo.forward(toks, bb.as_float(W), cfg)[0]
    model = zb.upload(ctx, cfg, W, F32)
    s = lva.Session(model, 32)
    s.begin(toks[:20], 0)
    s.wait()
    for p in range(20, 440):
        if p in (32, 48, 300):               # growing keeps what is there
            s.reserve({32: 48, 48: 300, 300: 600}[p])
        s.begin(toks[p:p + 1], p)
        if p % 13 == 0 or p > 430:
            assert rel(s.logits()[None], want[p:p + 1]) < 2e-4, p
        else:
            s.wait()
    assert s.position() == 440
    s.close()
    model.close()


# ---- keys and states that stand out ------------------------------------------------------------------------------------------
def beacon(n, asks, keys, seed=50, heads=3):
    """One layer of latent attention in which the tokens at `asks` carry a query that matches, at any distance, the key of the
    tokens at `keys` and nothing else: unrotated dimensions, scores around 30."""
    cfg = zb.config(vocab=40, width=64, streams=1, bigram=None, scale=1.0,
                    layers=[zb.layer(zb.latent(heads=heads, dim=16, rot_dim=8, vdim=16, q_rank=24, kv_rank=24, scale=1.0), 0)])
    W = zb.weights(cfg, seed)
    F = bb.as_float(W)
    E, p = F["embed"], "l0.mix."
    E[:, :2] = 0
    E[38], E[39] = 0, 0
    E[38, 0] = 6.0           # asks
    E[39, 1] = 6.0           # answers
    E[39, 2:] = np.random.default_rng(seed).standard_normal(62)
    F["l0.norm1"][:], F["l0.norm1.b"][:], F["l0.norm1.alpha"] = 1.0, 0.0, np.array(1.0)
    F["l0.hc1.in"][:], F["l0.hc1.out"][:], F["l0.hc1.mix"][:] = 1.0, 1.5, 1.0
    for r, col in (("dq", 0), ("dkv", 1)):
        F[p + r][:, :2] = 0
        F[p + r][0] = 0
        F[p + r][0, col] = 6.0                   # latent 0: this token asks / answers
        F[p + r + ".norm"][:] = 1.0
    F[p + "dq"][1:, 0] = 0
    F[p + "uq"][:, 0], F[p + "uk"][:, 0] = 0, 0
    F[p + "uq"] *= 0.3
    for h in range(heads):
        F[p + "uq"][h * 24] = 0
        F[p + "uk"][h * 16] = 0
        F[p + "uq"][h * 24, 0], F[p + "uk"][h * 16, 0] = 3.0, 3.0
    toks = np.random.default_rng(seed + 1).integers(0, 38, n).astype(np.uint32)
    toks[list(asks)] = 38
    toks[list(keys)] = 39
    return cfg, {name: bb.to_bf16(v).reshape(np.shape(v)) for name, v in F.items()}, toks


@pytest.mark.parametrize("compute", [F32, BF16])
@pytest.mark.parametrize("key", [0, 1, 31, 32, 63, 64, 127, 128, 129, 191, 300])
def test_a_far_key_among_hundreds(lva, ctx, key, compute):
    """one key at the edges of blocks, tiles and portions, asked for from right behind it, from edges, and from far away"""
    asks = {p for p in (key + 1, key + 2, 127, 128, 129, 130, 255, 256, 257, 320, 383, 384, 385, 450) if p > key}
    cfg, W, toks = beacon(460, asks, {key})
    F = bb.as_float(W)
    want = zo.forward(toks, F, cfg)[0]
    rows = sorted(asks)
    # the inputs tell: without the key, and without the sink, these rows would be far off
    i = np.arange(460)
    mask = i[None] <= i[:, None]
    mask[:, key] = i == key
    assert np.min(np.max(np.abs(zo.forward(toks, F, cfg, mask=mask)[0] - want), axis=1)[rows]) > 0.3
    with device(lva, ctx, cfg, W, compute) as d:
        for cuts in ((1000,), (120, 1), (200, 100, 2), (64,), (key + 1, 1) if key < 200 else (key + 1, 50)):
            assert rel(d.run(toks, cuts)[rows], want[rows]) < 2 * TOL[compute], cuts


@pytest.mark.parametrize("compute", [F32, BF16])
def test_the_sink_takes_its_share(lva, ctx, compute):
    """a sink as large as the best score halves the answer, and another head's sink would show"""
    cfg, W, toks = beacon(140, {20, 70, 139}, {3})
    F = bb.as_float(W)
    F["l0.mix.sink"][:] = [30.0, 33.0, -20.0]
    W["l0.mix.sink"] = bb.to_bf16(F["l0.mix.sink"])
    F = bb.as_float(W)
    want = zo.forward(toks, F, cfg)[0]
    assert np.max(np.abs(zo.forward(toks, F, cfg, with_sink=False)[0] - want)) > 0.3
    F["l0.mix.sink"] = F["l0.mix.sink"][::-1]
    assert np.max(np.abs(zo.forward(toks, F, cfg)[0] - want)) > 0.3
    with device(lva, ctx, cfg, W, compute) as d:
        for cuts in ((1000,), (1,), (17, 2)):
            assert rel(d.run(toks, cuts), want) < 2 * TOL[compute], cuts


def one_ssm(seed, **kw):
    cfg = zb.config(vocab=40, width=40, streams=1, bigram=None, layers=[zb.layer(zb.ssm(**{**dict(heads=4, groups=2, state=30, vdim=12, conv=4, norm_groups=2), **kw}), 0)])
    return cfg, zb.weights(cfg, seed)


@pytest.mark.parametrize("compute", [F32, BF16])
def test_the_recurrent_state_remembers(lva, ctx, compute):
    """a slow decay: the first token still shows after 200 others, through portions and decoding"""
    cfg, W = one_ssm(61)
    W["l0.mix.A_log"] = bb.to_bf16(np.full(4, -6.0))
    toks = tokens_for(cfg, 200, 6)
    F = bb.as_float(W)
    want = zo.forward(toks, F, cfg)[0]
    other = toks.copy()
    other[0] = (other[0] + 1) % 40
    assert np.max(np.abs(zo.forward(other, F, cfg)[0][-1] - want[-1])) > 2e-3 * np.max(np.abs(want[-1]))
    with device(lva, ctx, cfg, W, compute) as d:
        for cuts in ((1000,), (3, 100, 1), (64, 16, 2), (1,)):
            assert rel(d.run(toks, cuts), want) < TOL[compute], cuts


@pytest.mark.parametrize("compute", [F32, BF16])
def test_strong_and_small_decays(lva, ctx, compute):
    """heads that forget within a token beside heads whose rate is e^-9 times a large factor: what every token takes off the state
    has to be right, not only its absolute size"""
    cfg, W = one_ssm(67)
    W["l0.mix.dt_bias"] = bb.to_bf16(np.array([-9.0, 4.0, -9.0, 1.0]))
    W["l0.mix.A_log"] = bb.to_bf16(np.array([3.5, 4.0, 1.0, 2.0]))
    toks = tokens_for(cfg, 400, 8)
    want = zo.forward(toks, bb.as_float(W), cfg)[0]
    with device(lva, ctx, cfg, W, compute) as d:
        for cuts in ((1000,), (150, 1), (65, 2, 130)):
            assert rel(d.run(toks, cuts), want) < TOL[compute], cuts


# ---- sessions --------------------------------------------------------------------------------------------------------------
def test_a_session_used_again_and_sessions_side_by_side(lva, ctx):
    cfg = deep()
    W = zb.weights(cfg, 45)
    F = bb.as_float(W)
    a, b, c = (tokens_for(cfg, n, 70 + n) for n in (90, 23, 61))
    want = {id(t): zo.forward(t, F, cfg)[0] for t in (a, b, c)}
    with device(lva, ctx, cfg, W, F32) as d:
        first = d.run(a, (1000,))
        assert rel(first, want[id(a)]) < 1e-4
        # a shorter, then another sequence in the same rows and state
        assert rel(d.run(b, (2, 1)), want[id(b)]) < 1e-4
        assert rel(d.run(c, (30, 1, 16, 2)), want[id(c)]) < 1e-4
        assert np.array_equal(d.run(a, (1000,)), first)
        # a second session of the model, steps alternating
        e = lva.Session(d.model, 128)
        e.keep_all_logits(True)
        pos = {id(d.sess): 0, id(e): 0}
        for n in (20, 1, 2, 17, 1):
            for s, t in ((d.sess, a), (e, c)):
                p = pos[id(s)]
                s.begin(t[p:p + n], p)
                assert rel(s.logits_rows(0, n), want[id(t)][p:p + n]) < 1e-4
                pos[id(s)] = p + n
        e.close()


@pytest.mark.parametrize("at", [60, 61])
def test_state_goes_to_another_session(lva, ctx, at):
    """every pass's cache rows and state, and the last token"""
    cfg = deep()
    W = zb.weights(cfg, 47)
    toks = tokens_for(cfg, 80, 2)
    want = zo.forward(toks, bb.as_float(W), cfg)[0]
    with device(lva, ctx, cfg, W, F32) as d:
        d.run(toks[:at], (1000,))
        e = lva.Session(d.model, 64)
        e.begin([1, 2, 3], 0)
        e.wait()
        e.reserve(100)
        for i in range(len(zo.run_order(cfg))):
            e.state_write(i, at, d.sess.state(i, at))
        assert e.position() == at
        for p in range(at, 80):
            got = d.step(toks[p:p + 1], p)
            e.begin(toks[p:p + 1], p)
            assert np.array_equal(e.logits(), got[0]), p
            assert rel(got, want[p:p + 1]) < 1e-4
        e.close()


def test_bad_models_are_refused(lva, ctx):
    cfg = deep()
    W = zb.weights(cfg, 1)

    def refused(code, change_w=None, change_cfg=None):
        w, c = dict(W), json.loads(json.dumps(cfg))
        if change_w:
            change_w(w)
        if change_cfg:
            change_cfg(c)
        with pytest.raises(lva.LvError) as e:
            zb.upload(ctx, c, w, F32)
        assert e.value.code == code
        return str(e.value)
    for name in ("l1.mix.uv", "l0.mix.conv.b", "l3.hc2.mix", "bigram", "l0.norm2.alpha", "l0.mlp.down", "final.norm.b"):
        assert name in refused(-6, lambda w: w.pop(name))
        assert name in refused(-1, lambda w: w.update({name: np.zeros(np.array(w[name].shape, int) + 1, np.uint16) if w[name].ndim else np.zeros(2, np.uint16)}))
    refused(-1, change_cfg=lambda c: c["layers"][0]["mixer"].update(groups=2))
    refused(-1, change_cfg=lambda c: c["layers"][0]["mixer"].update(norm_groups=7))
    refused(-1, change_cfg=lambda c: c["layers"][0]["mixer"].update(state=257))
    refused(-1, change_cfg=lambda c: c["layers"][1]["mixer"]["rot"].update(dims=10))
    refused(-1, change_cfg=lambda c: c["layers"][1]["mixer"].update(dim=250))
    refused(-1, change_cfg=lambda c: c["layers"][1]["mixer"].update(kv_rank=800))
    refused(-1, change_cfg=lambda c: c.update(streams=9))
    refused(-1, change_cfg=lambda c: c["loop"].update(stop=6))
    refused(-1, change_cfg=lambda c: c["loop"].update(times=4000000000))


# ---- host classes, command line, trace runner --------------------------------------------------------------------------------
@pytest.fixture(scope="module")
def folder(tmp_path_factory):
    cfg = zb.config(vocab=61, width=48, streams=2, loop=(1, 3, 2))
    p = str(tmp_path_factory.mktemp("zedenex") / "model")
    return p, cfg, bb.write_folder(p, cfg, W=zb.weights(cfg, 82))


def clear_greedy(prompt, count, F, cfg):
    """greedy continuation; every choice has to be clear, so that rounding cannot turn one"""
    seq = list(prompt)
    for _ in range(count):
        z = np.sort(zo.forward(seq, F, cfg)[0][-1])
        assert z[-1] - z[-2] > 1e-3
        seq += zo.greedy(seq, 1, F, cfg)
    return seq[len(prompt):]


def test_greedy_generation_through_the_session_class(hostlib, folder):
    path, cfg, W = folder
    F = bb.as_float(W)
    prompt = [12, 7, 40, 44, 60, 0, 9, 12, 12, 30, 31, 7, 8, 55, 2, 19, 40, 41, 6]
    want = clear_greedy(prompt, 24, F, cfg)
    c = hostlib.LlavaContext()
    assert c.load_model(path, compute=F32), c.error()
    s = hostlib.LlavaSession(c)
    assert s.good() and s.layer_count() == 6
    assert s.set_text(" ".join(map(str, prompt)).encode())
    got = []
    for _ in range(24):
        got.append(s.predict(deterministic=True))
        assert s.push_token(got[-1])
    assert got == want
    # back in the sequence: the state is built again from the start
    s.rewind(len(prompt) + 5)
    assert s.tokens_in_gpu() == 0 and s.predict(True) == want[5]
    # more text goes on from where the state stands; other text starts anew
    at = s.tokens_in_gpu()
    assert s.add_text(b"4, 5") and s.tokens_in_gpu() == at
    assert s.predict(True) == zo.greedy(prompt + want[:5] + [4, 5], 1, F, cfg)[0]
    assert s.set_text(b"5 17 9") and s.tokens_in_gpu() == 0
    assert s.predict(True) == zo.greedy([5, 17, 9], 1, F, cfg)[0]
    s.close()
    c.close()


def test_snapshot_and_restore(hostlib, folder, tmp_path):
    path, cfg, W = folder
    c = hostlib.LlavaContext()
    assert c.load_model(path, compute=F32)
    toks = [int(t) for t in tokens_for(cfg, 151, 9)]
    a = hostlib.LlavaSession(c)
    assert a.push_tokens(toks)
    first = a.predict(True)
    f = str(tmp_path / "snap")
    assert a.snapshot(f) == hostlib.RC_OK
    b = hostlib.LlavaSession(c)
    assert b.push_tokens([1, 2, 3]) and b.predict(True) is not None
    assert b.restore(f) == hostlib.RC_OK and b.tokens() == toks and b.tokens_in_gpu() == 151
    for s in (a, b):
        assert s.push_token(first)
    for _ in range(5):
        x, y = a.predict(True), b.predict(True)
        assert x == y and np.array_equal(a.logits(), b.logits())
        assert a.push_token(x) and b.push_token(y)
    for s in (a, b):
        s.close()
    c.close()


def test_command_line_generates_ids(lva, folder):
    path, cfg, W = folder
    exe = os.path.join(lva.PKG_DIR, "bin", "llava")
    out = subprocess.run([exe, "-m", path, "--dtype", "float32", "--greedy", "-n", "6", "12 7 40"], capture_output=True, text=True, timeout=100)
    assert out.returncode == 0, out.stderr
    assert [int(t) for t in out.stdout.split()[:9]] == [12, 7, 40] + zo.greedy([12, 7, 40], 6, bb.as_float(W), cfg)


def test_token_server(hostlib, folder):
    path, cfg, W = folder
    c = hostlib.LlavaContext()
    assert c.load_model(path, compute=F32)
    server = hostlib.LlavaServer(c)
    a, b = sc.Client(server.port), sc.Client(server.port)
    F = bb.as_float(W)
    prompts = {}
    for client, text in ((a, b"12 7 40 9"), (b, b"44, 2")):      # two sessions, ticks in turn
        sid = client.new_session()
        assert client.ack(sc.SET_OPTIONS, sid, sc.OPTION_GREEDY) == sc.RC_OK
        assert client.ack(sc.ADD_TEXT, sid, text=text) == sc.RC_OK
        prompts[client] = (sid, client.tokens(sid))
    got = {client: [] for client in prompts}
    for _ in range(8):
        for client, (sid, _) in prompts.items():
            got[client].append(client.tick(sid)[0])
    for client, (sid, prompt) in prompts.items():
        assert got[client] == zo.greedy(prompt, 8, F, cfg)
        client.close()
    server.stop()
    c.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run(lva, folder, tmp_path, dtype):
    path, cfg, W = folder
    a, b = tokens_for(cfg, 60, 11), tokens_for(cfg, 9, 12)
    F = bb.as_float(W)
    steps = [dict(step=0, entries=[dict(id="a", tokens=a[:40].tolist(), want=[0, 39])], end=[]),
             dict(step=1, entries=[dict(id="b", tokens=b.tolist(), want=[8, 3])], end=["b"]),
             dict(step=2, entries=[dict(id="a", tokens=a[40:42].tolist(), want=[])], end=[]),
             dict(step=3, entries=[dict(id="a", tokens=a[42:].tolist(), want=[17])], end=["a"]),
             dict(step=4, entries=[dict(id="a", tokens=b[:1].tolist(), want=[0])], end=["a"])]
    exe = os.path.join(lva.ROOT_DIR, "bin", "trace_run")
    r = subprocess.run([exe, "--model", path, "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "200"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(5)]
    wa, wb = zo.forward(a, F, cfg)[0], zo.forward(b, F, cfg)[0]
    tol = {"float32": 1e-4, "bfloat16": 6e-2}[dtype]

    def rows(i):
        return np.fromfile(str(tmp_path / f"{i}.f32"), dtype="<f4").reshape(-1, cfg["vocab"])
    assert rel(rows(0), wa[[0, 39]]) < tol
    assert rel(rows(1), wb[[8, 3]]) < tol
    assert not (tmp_path / "2.f32").exists()
    assert rel(rows(3), wa[[59]]) < tol
    assert rel(rows(4), wb[[0]]) < tol
