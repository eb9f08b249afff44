#!/usr/bin/env python3
"""Measurements of the decode path beyond the headline bench: one JSON line per case.

    python llama-vulkan_amd/measure.py gemv          isolated dequant-fused GEMVs at the 7B shapes, q4_0 and q8_0
    python llama-vulkan_amd/measure.py attention     the one-token attention kernel by itself (7B heads) over 512 and 2048 cache rows
    python llama-vulkan_amd/measure.py decode-q8     7B q8_0, cache positions 1920..2047 (128 greedy steps)
    python llama-vulkan_amd/measure.py decode-q8-graph    the same on the hipGraph of the operator chain (attention_kernel over 2048 rows)
    python llama-vulkan_amd/measure.py gemv-13b      the same GEMVs at the 13B layer shapes
    python llama-vulkan_amd/measure.py decode-13b    13B q4_0, 32-token prompt + 256 greedy steps (persistent kernel)
    python llama-vulkan_amd/measure.py decode-13b-graph   the same on the hipGraph of the operator chain
    python llama-vulkan_amd/measure.py decode-7b-graph    7B q4_0, positions 444..511 on the hipGraph of the operator chain
    python llama-vulkan_amd/measure.py prefill-13b   13B q8_0, 512-token prompt evaluated in one lv_step_begin
    python llama-vulkan_amd/measure.py prefill-7b    7B q4_0, the same
    python llama-vulkan_amd/measure.py prefill-13b-q4  13B q4_0, the same
    python llama-vulkan_amd/measure.py gemm          isolated 512-token GEMMs at the 13B shapes, q8_0 (for kernel traces and counters)
    python llama-vulkan_amd/measure.py copy          1 GiB device-to-device copy: achievable bandwidth, counter calibration
    python llama-vulkan_amd/measure.py read-stream   4 GiB read by a kernel that only reads: the bandwidth a weight stream can reach
    python llama-vulkan_amd/measure.py block [SIZE]  block models beside LLaMA layers of the same width (bench.py --block)
    python llama-vulkan_amd/measure.py zedenex [SIZE]    Zedenex beside Somesun of the same width (bench.py --block Zedenex)
    python llama-vulkan_amd/measure.py block-only SIZE   prompts and decode steps of Somesun alone (for kernel traces); zedenex-only SIZE: of Zedenex
    python llama-vulkan_amd/measure.py all

Every figure is algorithmic bytes (weights as stored in the GGML file, 18 B / 34 B per 32 weights, plus vectors and the
fp16 cache rows a step reads) divided by the time measured with HIP events on the stream that runs the kernels.
Models are seeded synthetic GGJT files written to /dev/shm (or /tmp) on first use.  Every case function returns its
figures as a dict (bench.py collects them under "cases"); run as a script, each is printed as one JSON line."""
import importlib
import json
import os
import sys
import time

HERE = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, os.path.dirname(HERE))
lva = importlib.import_module("llama-vulkan_amd")
HBM_PEAK_GBS = 8000.0
SHAPES = {"7b": dict(vocab=32000, dim=4096, heads=32, layers=32, ff=11008), "13b": dict(vocab=32000, dim=5120, heads=40, layers=40, ff=13824)}


def emit(**kw):
    print(json.dumps({k: v for k, v in kw.items() if k != "picks"}), flush=True)
    return kw


def block_bytes(ftype):
    return 18 if ftype == lva.LV_Q4_0 else 34


GEMV_SHAPES_7B = ((4096, 4096, "store"), (11008, 4096, "silu"), (4096, 11008, "add"), (32000, 4096, "store"))
GEMV_SHAPES_13B = ((5120, 5120, "store"), (13824, 5120, "silu"), (5120, 13824, "add"), (32000, 5120, "store"))


def gemv_cases(ctx, report=emit, shapes=GEMV_SHAPES_7B):
    """reference: matmul.glsl / matmul_q8.glsl / matmul_silu_ff.comp at the three layer shapes and the output matrix"""
    out_cases = []
    for ftype, tname in ((lva.LV_Q4_0, "q4_0"), (lva.LV_Q8_0, "q8_0")):
        for rows, cols, mode in shapes:
            nbytes = rows * cols // 32 * block_bytes(ftype) * (2 if mode == "silu" else 1) + 4 * cols + 4 * rows * (2 if mode == "add" else 1)
            # enough distinct matrices that the working set exceeds the 256 MB last-level cache
            nmat = max(2, min(12, int(1.5e9 // nbytes)))
            mats = []
            for i in range(nmat * (2 if mode == "silu" else 1)):
                mats.append(ctx.matrix(lva.synth_quant(ftype, rows, cols, seed=100 + i), ftype, rows, cols))
            x = ctx.to_device(lva.synth_normal(1, cols, seed=1))
            out = ctx.zeros(rows * 4)

            def run(i):
                if mode == "silu":
                    lva.check(ctx.lib.lv_kernel_gemv_silu(ctx.h, out, mats[2 * i], mats[2 * i + 1], x, 1))
                else:
                    lva.check(ctx.lib.lv_kernel_gemv(ctx.h, out, mats[i], x, 1, 1 if mode == "add" else 0))
            for i in range(nmat):
                run(i)
            ctx.sync()
            iters = 20
            ctx.timer_start()
            for _ in range(iters):
                for i in range(nmat):
                    run(i)
            us = ctx.timer_stop() * 1e3 / (iters * nmat)
            out_cases.append(report(case="gemv", wtype=tname, rows=rows, cols=cols, mode=mode, us=round(us, 2), algorithmic_bytes=nbytes,
                                    GBps=round(nbytes / us / 1e3, 1), frac_of_peak=round(nbytes / us / 1e3 / HBM_PEAK_GBS, 4)))
            for m in mats:
                ctx.matrix_free(m)
            ctx.free(x)
            ctx.free(out)
    return out_cases


def quiet(**kw):
    return kw


def attention_cases(ctx, report=emit):
    """reference: mhsa.comp + softmax.comp + kqv_matching.comp for one query.  32 heads of 128 at the last row of a 512- and
    of a 2048-row cache; algorithmic bytes = the fp16 K and V rows 0..pos (4 * (pos + 1) * dim bytes) plus q in and out.
    Sixteen caches in turn (0.5 / 2 GB), so that the rows come from HBM."""
    import numpy as np
    out_cases = []
    heads, rot = 32, 128
    dim = heads * rot
    for backlog in (512, 2048):
        pos = backlog - 1
        ncache = 16
        rng = np.random.default_rng(backlog)
        host = (rng.standard_normal((backlog, dim)) * 0.5).astype(np.float16)
        ks = [ctx.to_device(host) for _ in range(ncache)]
        vs = [ctx.to_device(host) for _ in range(ncache)]
        q = ctx.to_device(lva.synth_normal(1, dim, seed=3))
        out = ctx.zeros(dim * 4)
        for i in range(ncache):
            lva.check(ctx.lib.lv_kernel_attention(ctx.h, out, ks[i], vs[i], q, pos, backlog, heads, rot, 1))
        ctx.sync()
        iters = 20
        ctx.timer_start()
        for _ in range(iters):
            for i in range(ncache):
                lva.check(ctx.lib.lv_kernel_attention(ctx.h, out, ks[i], vs[i], q, pos, backlog, heads, rot, 1))
        us = ctx.timer_stop() * 1e3 / (iters * ncache)
        nbytes = 4 * (pos + 1) * dim + 8 * dim
        out_cases.append(report(case="attention", heads=heads, head_size=rot, rows=pos + 1, us=round(us, 2), algorithmic_bytes=nbytes,
                                GBps=round(nbytes / us / 1e3, 1), frac_of_peak=round(nbytes / us / 1e3 / HBM_PEAK_GBS, 4)))
        for b in ks + vs + [q, out]:
            ctx.free(b)
    return out_cases


def attention_batch_cases(ctx, report=emit):
    """The prompt form of the same chain (lv_kernel_attention with 16 rows or more: attention_prepare_kernel, then
    attention_batch_kernel): n query rows at cache positions pos .. pos+n-1, 13B and 7B head counts.  Useful flops =
    4 * head_size * sum over the rows of the positions each sees (scores and sums, a multiply-add = 2); the kernels execute 4 x
    that (3 + 5 products of 16-bit operand pieces)."""
    import numpy as np
    out_cases = []
    rot = 128
    for heads, pos, n in ((40, 0, 512), (32, 0, 512), (40, 1536, 512), (40, 0, 128)):
        dim, backlog = heads * rot, 2048
        rng = np.random.default_rng(heads + pos)
        host = (rng.standard_normal((backlog, dim)) * 0.5).astype(np.float16)
        k, v = ctx.to_device(host), ctx.to_device(host)
        q = ctx.to_device(lva.synth_normal(n, dim, seed=3))
        out = ctx.zeros(n * dim * 4)
        for _ in range(3):
            lva.check(ctx.lib.lv_kernel_attention(ctx.h, out, k, v, q, pos, backlog, heads, rot, n))
        ctx.sync()
        iters = 50
        ctx.timer_start()
        for _ in range(iters):
            lva.check(ctx.lib.lv_kernel_attention(ctx.h, out, k, v, q, pos, backlog, heads, rot, n))
        us = ctx.timer_stop() * 1e3 / iters
        pairs = sum(pos + z + 1 for z in range(n))
        flops = 4.0 * rot * pairs * heads
        out_cases.append(report(case="attention-batch", heads=heads, head_size=rot, first_position=pos, rows=n, us_both_kernels=round(us, 2),
                                useful_TFLOPs=round(flops / us / 1e6, 1), executed_TFLOPs=round(4 * flops / us / 1e6, 1)))
        for b in (k, v, q, out):
            ctx.free(b)
    return out_cases


def copy_case(ctx):
    n = 1 << 30
    src, dst = ctx.zeros(n), ctx.zeros(n)
    lva.check(ctx.lib.lv_dev_copy(ctx.h, dst, src, n))
    ctx.sync()
    ctx.timer_start()
    for _ in range(4):
        lva.check(ctx.lib.lv_dev_copy(ctx.h, dst, src, n))
    ms = ctx.timer_stop() / 4
    emit(case="copy", bytes_read=n, bytes_written=n, ms=round(ms, 4), GBps_read_plus_write=round(2 * n / ms / 1e6, 1))
    ctx.free(src)
    ctx.free(dst)


def read_stream_case(ctx, report=emit, gib=4):
    """What a kernel that only reads memory reaches on this device (lv_dev_read: contiguous share per workgroup, 16-byte
    non-temporal loads, eight in flight): a buffer far larger than the 256 MB last-level cache, read 8 times.  The decode
    kernel's bytes per second are reported against this figure as well as against the 8 TB/s of the datasheet."""
    n = gib << 30
    src = ctx.zeros(n)
    lva.check(ctx.lib.lv_dev_read(ctx.h, src, n))
    ctx.sync()
    reps = 8
    ctx.timer_start()
    for _ in range(reps):
        lva.check(ctx.lib.lv_dev_read(ctx.h, src, n))
    ms = ctx.timer_stop() / reps
    ctx.free(src)
    return report(case="read-stream", bytes_read=n, ms=round(ms, 4), GBps=round(n / ms / 1e6, 1), frac_of_peak=round(n / ms / 1e6 / HBM_PEAK_GBS, 4))


def model_file(preset, wtype, seed):
    base = "/dev/shm" if os.access("/dev/shm", os.W_OK) else "/tmp"
    path = os.path.join(base, f"llava_measure_{preset}_{'q4_0' if wtype == lva.LV_Q4_0 else 'q8_0'}_seed{seed}.ggml")
    if (preset, wtype, seed) == ("7b", lva.LV_Q4_0, 0):
        path = os.path.join(base, "llava_bench_7b_q4_0_seed0.ggml")      # the file bench.py and the full-size tests use
    if not os.path.exists(path):
        lva.write_model(path + ".tmp", wtype=wtype, seed=seed, **SHAPES[preset])
        os.replace(path + ".tmp", path)
    return path


def step_bytes(shape, wtype, pos):
    D, F, V, L = shape["dim"], shape["ff"], shape["vocab"], shape["layers"]
    per_layer = (4 * D * D + 3 * D * F) // 32 * block_bytes(wtype)
    return L * per_layer + V * D // 32 * block_bytes(wtype) + (2 * L + 1) * D * 4 + L * 2 * D * 2 * (pos + 2) + V * 4 + D * 4


def decode_case(ctx, name, preset, wtype, seed, backlog, first, steps, force_path=None, report=emit, expect_picks=None):
    shape = SHAPES[preset]
    path = model_file(preset, wtype, seed)
    model = lva.Model(ctx, path)
    s = lva.Session(model, backlog)
    if force_path is not None:
        s.set_path(force_path)
    kind = {lva.PATH_KERNELS: "kernels", lva.PATH_GRAPH: "graph", lva.PATH_PERSISTENT: "persistent"}[s.path()]
    prompt = lva.synth_tokens(first, 3, shape["vocab"], seed=seed)
    t0 = time.perf_counter()
    s.begin(prompt, 0)
    tok = s.argmax()
    prefill_s = time.perf_counter() - t0
    pos = first
    picks = [tok]                      # picks[k] is the token fed at position first + k
    for _ in range(4):
        s.begin([tok], pos)
        tok = s.argmax()
        picks.append(tok)
        pos += 1
    t0 = time.perf_counter()
    total = 0
    for _ in range(steps):
        s.begin([tok], pos)
        tok = s.argmax()
        picks.append(tok)
        total += step_bytes(shape, wtype, pos)
        pos += 1
    dt = time.perf_counter() - t0
    if expect_picks is not None:       # another path's run of the same case: the greedy continuation has to be the same
        n = min(len(expect_picks), len(picks))
        diff = [k for k in range(n) if picks[k] != expect_picks[k]]
        if diff:
            raise RuntimeError(f"{name}: greedy token at position {first + diff[0]} differs from the other path's ({picks[diff[0]]} vs {expect_picks[diff[0]]})")
    r = report(case=name, model=preset, wtype="q4_0" if wtype == lva.LV_Q4_0 else "q8_0", path=kind, positions=[first + 4, pos - 1], steps=steps,
               tok_s=round(steps / dt, 1), ms_per_token=round(dt / steps * 1e3, 4), GBps=round(total / dt / 1e9, 1),
               frac_of_peak=round(total / dt / 1e9 / HBM_PEAK_GBS, 4), prompt_tokens=first, prompt_s=round(prefill_s, 3),
               same_picks_as_other_path=None if expect_picks is None else True)
    s.close()
    model.close()
    r = dict(r)
    r["picks"] = picks
    return r


MFMA_PEAK_TFLOPS = 2500.0


def prefill_case(ctx, case, name, wtype, report=emit):
    shape = SHAPES[name]
    path = model_file(name, wtype, 3)
    model = lva.Model(ctx, path)
    s = lva.Session(model, 512)
    prompt = lva.synth_tokens(512, 3, shape["vocab"], seed=3)
    s.begin(prompt, 0)          # untimed: allocates the prompt workspace and makes the model's prompt copy
    s.wait()
    s.timer_start()
    s.begin(prompt, 0)          # the same rows again
    ms = s.timer_stop()
    D, F, V, L = shape["dim"], shape["ff"], shape["vocab"], shape["layers"]
    flops = 2.0 * 512 * L * (4 * D * D + 3 * D * F) + 2.0 * V * D      # the output matrix sees the last row only
    # frac_of_mfma_peak counts the flops the prompt needs (2 per weight and token); the GEMM executes every product twice
    # (activations are a pair of fp16 halves), so the matrix cores run at twice that rate: executed_frac
    r = report(case=case, model=name, wtype="q4_0" if wtype == lva.LV_Q4_0 else "q8_0", tokens=512, ms=round(ms, 2),
               tok_s=round(512 / ms * 1e3, 1), TFLOPs=round(flops / ms / 1e9, 2), executed_TFLOPs=round(2 * flops / ms / 1e9, 2),
               frac_of_mfma_peak=round(flops / ms / 1e9 / MFMA_PEAK_TFLOPS, 4), executed_frac=round(2 * flops / ms / 1e9 / MFMA_PEAK_TFLOPS, 4))
    s.close()
    model.close()
    return r


def gemm_cases(ctx, report=emit):
    """reference: the *_batch shaders on 512 pending tokens (llava_session.cpp:243-255).  One lv_kernel_gemm call = the split of
    the activations into fp16 halves + gemm_kernel (+ the sum of the K slices where the grid would not fill the device), at
    the 13B layer shapes; the matrix's prompt copy and the workspace exist after the first call.  flops = 2 * tokens *
    rows * cols; every product is executed twice (two activation halves)."""
    n, wtype = 512, lva.LV_Q8_0
    out_cases = []
    for rows, cols in ((5120, 5120), (13824, 5120), (5120, 13824)):
        m = ctx.matrix(lva.synth_quant(wtype, rows, cols, seed=1), wtype, rows, cols)
        x = ctx.to_device(lva.synth_normal(n, cols, seed=2))
        out = ctx.zeros(n * rows * 4)
        for _ in range(3):
            lva.check(ctx.lib.lv_kernel_gemm(ctx.h, out, m, x, n, 0))
        ctx.sync()
        reps = 20
        ctx.timer_start()
        for _ in range(reps):
            lva.check(ctx.lib.lv_kernel_gemm(ctx.h, out, m, x, n, 0))
        us = ctx.timer_stop() * 1e3 / reps
        useful = 2.0 * n * rows * cols / us / 1e6
        out_cases.append(report(case="gemm", wtype="q8_0", rows=rows, cols=cols, tokens=n, launches=reps, us=round(us, 1),
                                useful_TFLOPs=round(useful, 1), executed_TFLOPs=round(2 * useful, 1),
                                frac_of_mfma_peak=round(useful / MFMA_PEAK_TFLOPS, 4), executed_frac=round(2 * useful / MFMA_PEAK_TFLOPS, 4)))
        ctx.matrix_free(m)
        ctx.free(x)
        ctx.free(out)
    return out_cases


# Block models of the Somesun design at the layer sizes of real models, next to LLaMA layers of the same width and a like number
# of weights a token passes through
BLOCK_SIZES = {
    "4096": dict(vocab=32000, width=4096, layers=4, attn=(32, 8, 128, 8192), delta=(32, 16, 128, 128, 4), rank=128, moe=(64, 8, 1024),
                 llama=dict(vocab=32000, dim=4096, heads=32, layers=4, ff=11008)),
    "2048": dict(vocab=32000, width=2048, layers=6, attn=(16, 4, 128, 2048), delta=(16, 16, 128, 128, 4), rank=64, moe=(32, 4, 1024),
                 llama=dict(vocab=32000, dim=2048, heads=16, layers=6, ff=5504)),
}


def block_model(ctx, size, compute=None):
    """random weights: every matrix reads the same random bytes of host memory and gets its own place on the device, norm weights
    are ones"""
    import numpy as np
    c = BLOCK_SIZES[size]
    D, V, L, r = c["width"], c["vocab"], c["layers"], c["rank"]
    H, G, d, chunk = c["attn"]
    dh, dg, dk, dv, taps = c["delta"]
    E, top, ff = c["moe"]
    blob = max(V, H * d, dh * dv, ff) * max(D, H * d, dh * dv, ff)
    rng = np.random.default_rng(7)
    x = np.tile((rng.standard_normal(1 << 22) * 0.02).astype(np.float32), (blob + (1 << 22) - 1) >> 22)[:blob]
    ones = max(D, H * d, dh * dk)
    base = np.concatenate([(x.view(np.uint32) >> 16).astype(np.uint16), np.full(ones, 0x3F80, np.uint16)])
    table = []

    def t(name, rows, cols=1, one=False):
        table.append((name, lva.LV_BF16, blob * 2 if one else 0, rows, cols, rows * cols * 2))
    t("embed", V, D); t("head", V, D); t("final.norm", D, one=True)
    for i in range(L):
        p = f"l{i}."
        for n in ("norm1", "norm1b", "norm2", "norm2b"):
            t(p + n, D, one=True)
        a = p + "mix.left."
        t(a + "q", H * d, D); t(a + "k", G * d, D); t(a + "o", D, H * d); t(a + "sink", H)
        t(a + "q.norm", H * d, one=True); t(a + "k.norm", G * d, one=True)
        a = p + "mix.right."
        for n, rows in (("q", dg * dk), ("k", dg * dk), ("v", dh * dv)):
            t(a + n, rows, D); t(a + n + ".conv", rows, taps)
        t(a + "b", dh, D); t(a + "a1", r, D); t(a + "a2", dh * dk, r); t(a + "g1", r, D); t(a + "g2", dh * dv, r)
        t(a + "A_log", dh); t(a + "dt_bias", dh * dk); t(a + "norm", dv, one=True); t(a + "o", D, dh * dv)
        t(p + "mlp.router", E, D)
        for e in range(E):
            t(f"{p}mlp.e{e}.gate", ff, D); t(f"{p}mlp.e{e}.up", ff, D); t(f"{p}mlp.e{e}.down", D, ff)
    b = lva.BlockSpec()
    b.attn_scale, b.delta_scale = 0.7, 0.7
    b.attn = lva.AttnSpec(H, G, d, d, d ** -0.5, chunk, d, 500000.0, lva.ATTN_NORM_FULL | lva.ATTN_KEYS_AS_VALUES | lva.ATTN_SINK)
    b.delta = lva.DeltaSpec(dh, dg, dk, dv, taps)
    b.moe = lva.MoeSpec(E, top, ff)
    return lva.BlockModel(ctx, base.view(np.uint8), table, [b] * L, V, D, 1e-5, lva.LV_BF16 if compute is None else compute)


def block_step_cost(c, pos):
    """bytes a decode step at position `pos` has to move (bf16 weights of what the token passes through, the chunk's cache rows, the
    recurrent state in and out) and flops per token of a prompt (products with weights only)"""
    D, V, L, r = c["width"], c["vocab"], c["layers"], c["rank"]
    H, G, d, chunk = c["attn"]
    dh, dg, dk, dv, _ = c["delta"]
    E, top, ff = c["moe"]
    w = D * (H * d + G * d + 2 * dg * dk + dh * dv + dh + 2 * r) + r * dh * (dk + dv) + D * (H * d + dh * dv) + E * D + top * 3 * ff * D
    state = 2 * G * d * 2 * (pos % chunk + 1) + 2 * dh * dk * dv * 4
    return L * (2 * w + state) + 2 * V * D, 2.0 * L * w


# Zedenex at layer sizes of real models: latent attention with a dense feed-forward behind it, and state-space layers without one;
# compared with Somesun of the same width above
ZEDENEX_SIZES = {
    "4096": dict(vocab=32000, width=4096, streams=4, latent=(32, 128, 64, 128, 1536, 512), ssm=(128, 8, 128, 64, 4), ff=11008, layers="LMLM"),
    "2048": dict(vocab=32000, width=2048, streams=2, latent=(16, 128, 64, 128, 768, 512), ssm=(64, 1, 128, 64, 4), ff=5504, layers="LMLMLM"),
}


def zedenex_model(ctx, size, compute=None):
    """random weights, as block_model has them: matrices share random bytes on the host; a layer "L" is latent attention with its
    feed-forward, "M" a state-space layer"""
    import numpy as np
    c = ZEDENEX_SIZES[size]
    D, V, S, ff = c["width"], c["vocab"], c["streams"], c["ff"]
    H, d, r, vd, qr, kr = c["latent"]
    mh, g, n, mv, taps = c["ssm"]
    inner, chan = mh * mv, mh * mv + 2 * g * n
    blob = max(V * D, ff * D, (inner + chan + mh) * D, H * (d + r) * qr)
    rng = np.random.default_rng(7)
    x = np.tile((rng.standard_normal(1 << 22) * 0.02).astype(np.float32), (blob + (1 << 22) - 1) >> 22)[:blob]
    ones = max(D, inner, qr, kr)
    base = np.concatenate([(x.view(np.uint32) >> 16).astype(np.uint16), np.full(ones, 0x3F80, np.uint16)])
    table, blocks = [], []

    def t(name, rows, cols=1, one=False):
        table.append((name, lva.LV_BF16, blob * 2 if one else 0, rows, cols, rows * cols * 2))

    def site(norm, hc):
        t(norm, D, one=True); t(norm + ".b", D); t(norm + ".alpha", 1, one=True)
        if hc:
            t(hc + "in", S, one=True); t(hc + "out", S, one=True); t(hc + "mix", S, S)
    t("embed", V, D); t("bigram", 4098, D); site("final.norm", None)
    for i, kind in enumerate(c["layers"]):
        p, m, b = f"l{i}.", f"l{i}.mix.", lva.BlockSpec()
        site(p + "norm1", p + "hc1.")
        if kind == "L":
            site(p + "norm2", p + "hc2.")
            t(m + "dq", qr, D); t(m + "dq.norm", qr, one=True); t(m + "uq", H * (d + r), qr); t(m + "dkv", kr + r, D); t(m + "dkv.norm", kr, one=True)
            t(m + "uk", H * d, kr); t(m + "uv", H * vd, kr); t(m + "sink", H); t(m + "o", D, H * vd)
            t(p + "mlp.gate", ff, D); t(p + "mlp.up", ff, D); t(p + "mlp.down", D, ff)
            b.latent = lva.LatentSpec(H, d, r, vd, qr, kr, (d + r) ** -0.5, r, 10000.0, lva.ATTN_SINK)
            b.dense = lva.DenseSpec(ff, lva.ACT_RELU)
        else:
            t(m + "in", inner + chan + mh, D); t(m + "conv", chan, taps); t(m + "conv.b", chan); t(m + "dt_bias", mh); t(m + "A_log", mh); t(m + "D", mh)
            t(m + "norm", inner, one=True); t(m + "o", D, inner)
            b.ssm = lva.SsmSpec(mh, g, n, mv, taps, g)
        blocks.append(b)
    return lva.BlockModel(ctx, base.view(np.uint8), table, blocks, V, D, 1e-5, lva.LV_BF16 if compute is None else compute, norm=lva.NORM_TANH, streams=S,
                          tied_head=1, embed_scale=8.0, bigram_buckets=4097, bigram_prev=31, bigram_cur=17)


def zedenex_step_cost(c, pos):
    """as block_step_cost: a decode step reads the weights of every product once (W_uk as its transpose), the cache rows and the
    recurrent state; a prompt's token goes through every weight once"""
    D, V, ff = c["width"], c["vocab"], c["ff"]
    H, d, r, vd, qr, kr = c["latent"]
    mh, g, n, mv, _ = c["ssm"]
    inner, chan = mh * mv, mh * mv + 2 * g * n
    wl = D * (qr + kr + r) + H * (d + r) * qr + H * (d + vd) * kr + D * H * vd + 3 * D * ff
    wm = D * (inner + chan + mh) + D * inner
    nl, nm = c["layers"].count("L"), c["layers"].count("M")
    return nl * (2 * wl + 2 * (kr + r) * (pos + 1)) + nm * (2 * wm + 8 * inner * n) + 2 * V * D, 2.0 * (nl * wl + nm * wm)


def prompt_and_decode(s, vocab, label, cost, flops_per_token, report, prompts=(512, 2048), steps=64, **kw):
    """one model's prompts (each third run timed, with HIP events) and decode steps (wall clock, greedy pick included)"""
    out, n_max = [], max(prompts)
    for n in prompts:
        toks = lva.synth_tokens(n, 3, vocab, seed=n)
        for _ in range(2):
            s.begin(toks, 0)
            s.wait()
        s.timer_start()
        s.begin(toks, 0)
        ms = s.timer_stop()
        tf = flops_per_token * n / ms / 1e9
        out.append(report(case=label + " prompt", tokens=n, ms=round(ms, 3), tok_s=round(n / ms * 1e3, 1), TFLOPs=round(tf, 1),
                          frac_of_mfma_peak=round(tf / MFMA_PEAK_TFLOPS, 4), **kw))
    s.begin(lva.synth_tokens(n_max, 3, vocab, seed=1), 0)
    tok, pos, total = s.argmax(), n_max, 0
    for i in range(8 + steps):
        if i == 8:
            t0 = time.perf_counter()
        s.begin([tok], pos)
        tok = s.argmax()
        total += cost(pos) if i >= 8 else 0
        pos += 1
    dt = time.perf_counter() - t0
    out.append(report(case=label + " decode", positions=[n_max + 8, pos - 1], tok_s=round(steps / dt, 1), ms=round(dt / steps * 1e3, 4),
                      GBps=round(total / dt / 1e9, 1), frac_of_hbm_peak=round(total / dt / 1e9 / HBM_PEAK_GBS, 4), **kw))
    return out


def zedenex_cases(ctx, report=emit, sizes=None):
    """prefill and decode of Zedenex and of Somesun at the same width, same machine, same clock"""
    out = []
    for size in sizes or ZEDENEX_SIZES:
        for label, sizes_of, make, cost in ((f"Zedenex width {size}", ZEDENEX_SIZES, zedenex_model, zedenex_step_cost), (f"Somesun width {size}", BLOCK_SIZES, block_model, block_step_cost)):
            c = sizes_of[size]
            m = make(ctx, size)
            s = lva.Session(m, 2048 + 64 + 16)
            out += prompt_and_decode(s, c["vocab"], label, lambda pos: cost(c, pos)[0], cost(c, 0)[1], report, layers=len(c["layers"]) if isinstance(c["layers"], str) else c["layers"])
            s.close()
            m.close()
    return out


def block_cases(ctx, report=emit, sizes=None):
    """prefill and decode of a block model and of its LLaMA counterpart (q8_0, on the persistent kernel where it has one and on the
    graph of single kernels), same machine, same clock"""
    out_cases = []
    for size in sizes or BLOCK_SIZES:
        c = BLOCK_SIZES[size]
        m = block_model(ctx, size)
        s = lva.Session(m, 2048 + 64 + 16)
        _, fl = block_step_cost(c, 0)
        out_cases += prompt_and_decode(s, c["vocab"], f"Somesun width {size}", lambda pos: block_step_cost(c, pos)[0], fl, report, layers=c["layers"])
        s.close()
        m.close()
        L = c["llama"]
        base = "/dev/shm" if os.access("/dev/shm", os.W_OK) else "/tmp"
        path = os.path.join(base, f"llava_measure_block_{size}.ggml")
        if not os.path.exists(path):
            lva.write_model(path + ".tmp", wtype=lva.LV_Q8_0, seed=5, **L)
            os.replace(path + ".tmp", path)
        lm = lva.Model(ctx, path)
        s = lva.Session(lm, 2048 + 64 + 16)
        kinds = [lva.PATH_PERSISTENT, lva.PATH_GRAPH] if s.path() == lva.PATH_PERSISTENT else [lva.PATH_GRAPH]
        for k in kinds:
            s.set_path(k)
            out_cases += prompt_and_decode(s, L["vocab"], f"LLaMA width {size} q8_0, {'persistent' if k == lva.PATH_PERSISTENT else 'graph'}",
                                           lambda pos: step_bytes(L, lva.LV_Q8_0, pos), 2.0 * L["layers"] * (4 * L["dim"] ** 2 + 3 * L["dim"] * L["ff"]), report, layers=L["layers"])
        s.close()
        lm.close()
    return out_cases


def main():
    which = sys.argv[1] if len(sys.argv) > 1 else "all"
    ctx = lva.Context(0)
    name, cus, hbm = ctx.info()
    emit(case="device", name=name, compute_units=cus, hbm_GiB=hbm >> 30)
    if which in ("copy", "all"):
        copy_case(ctx)
    if which in ("read-stream", "all"):
        read_stream_case(ctx)
    if which in ("gemv", "all"):
        gemv_cases(ctx)
    if which == "gemv-13b":
        gemv_cases(ctx, shapes=GEMV_SHAPES_13B)
    if which in ("attention", "all"):
        attention_cases(ctx)
    if which == "attention-batch":
        attention_batch_cases(ctx)
    if which == "gemm":
        gemm_cases(ctx)
    if which == "block":
        block_cases(ctx, sizes=sys.argv[2:3] or None)
    if which == "zedenex":
        zedenex_cases(ctx, sizes=sys.argv[2:3] or None)
    if which in ("block-only", "zedenex-only"):     # one model by itself, for kernel traces: prompts of 2048, then decode
        c = (BLOCK_SIZES if which == "block-only" else ZEDENEX_SIZES)[sys.argv[2]]
        m = (block_model if which == "block-only" else zedenex_model)(ctx, sys.argv[2])
        s = lva.Session(m, 2200)
        toks = lva.synth_tokens(2048, 3, c["vocab"], seed=1)
        for _ in range(3):
            s.begin(toks, 0)
            s.wait()
        for pos in range(2048, 2080):
            s.begin([5], pos)
            s.wait()
        s.close()
        m.close()
    if which in ("decode-q8", "all"):
        decode_case(ctx, "decode-q8", "7b", lva.LV_Q8_0, 1, 2048, 1916, 128)
    if which in ("decode-q8-graph", "all"):
        decode_case(ctx, "decode-q8-graph", "7b", lva.LV_Q8_0, 1, 2048, 1916, 128, force_path=lva.PATH_GRAPH)
    if which in ("decode-13b", "all"):
        decode_case(ctx, "decode-13b", "13b", lva.LV_Q4_0, 2, 512, 32, 256)
    if which in ("decode-13b-graph", "all"):
        decode_case(ctx, "decode-13b-graph", "13b", lva.LV_Q4_0, 2, 512, 32, 256, force_path=lva.PATH_GRAPH)
    if which in ("decode-7b-graph", "all"):
        decode_case(ctx, "decode-7b-graph", "7b", lva.LV_Q4_0, 0, 512, 440, 68, force_path=lva.PATH_GRAPH)
    if which in ("prefill-13b", "all"):
        prefill_case(ctx, "prefill-13b", "13b", lva.LV_Q8_0)
    if which in ("prefill-13b-q4", "all"):
        prefill_case(ctx, "prefill-13b-q4", "13b", lva.LV_Q4_0)
    if which in ("prefill-7b", "all"):
        prefill_case(ctx, "prefill-7b", "7b", lva.LV_Q4_0)
    ctx.close()       # nothing of the library is left to the interpreter's exit


if __name__ == "__main__":
    main()
