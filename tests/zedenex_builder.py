"""Small random Zedenex models for the tests, and the same mechanisms put together otherwise: configurations, weights (bf16-exact),
and direct uploads through the C-ABI."""
import importlib

import numpy as np

import block_builder as bb


def latent(heads=3, dim=12, rot_dim=6, vdim=10, q_rank=20, kv_rank=18, base=700.0, scale=None):
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
            "rot": {"base": base, "dims": rot_dim}, "scale": (dim + rot_dim) ** -0.5 if scale is None else scale}


def ssm(heads=6, groups=3, state=20, vdim=7, conv=3, norm_groups=2):
    return {"heads": heads, "groups": groups, "state": state, "vdim": vdim, "conv": conv, "norm_groups": norm_groups}


def layer(mixer=None, ff=28):
    mixer = mixer or latent()
    return {"type": "latent_attention" if "kv_rank" in mixer else "mamba2", "mixer": mixer, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(vocab=53, width=44, streams=3, layers=None, loop=None, scale=5.5, bigram=(31, 7, 3), eps=1e-5):
    c = {"architecture": "Zedenex", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps},
         "embedding": {"scale": scale}, "layers": layers or [layer(), layer(ssm(), 0), layer(ssm(heads=2, groups=1)), layer(latent(heads=1), 0)]}
    if bigram:
        c["embedding"]["bigram"] = {"buckets": bigram[0], "mul_prev": bigram[1], "mul_cur": bigram[2]}
    if loop:
        c["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return c


def weights(cfg, seed, tanh=True, sinks=True, tied=True):
    """name -> bf16 bits.  tanh: norms are tanh norms, else RMS norms; without streams sublayers get a norm on their output"""
    rng = np.random.default_rng(seed)
    D, S, W = cfg["width"], cfg["streams"], {}

    def mat(name, rows, cols, gain=1.0):
        W[name] = rng.standard_normal((rows, cols)) * gain / np.sqrt(cols)

    def vec(name, n, mean=1.0, spread=0.2):
        W[name] = mean + spread * rng.standard_normal(n)

    def norm(name):
        vec(name, D)
        if tanh:
            vec(name + ".b", D, 0.0, 0.2)
            W[name + ".alpha"] = np.array(rng.uniform(0.3, 0.9))

    scale = cfg["embedding"]["scale"] or 1.0
    W["embed"] = rng.standard_normal((cfg["vocab"], D)) / scale
    if "bigram" in cfg["embedding"]:
        W["bigram"] = rng.standard_normal((cfg["embedding"]["bigram"]["buckets"] + 1, D)) * 0.7
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        for q in (1, 2) if l["mlp"] else (1,):
            norm(f"{p}norm{q}")
            if S:
                hc = f"{p}hc{q}."
                vec(hc + "in", S, 1.0 / S, 0.4)
                vec(hc + "out", S, 0.8, 0.4)
                W[hc + "mix"] = 0.8 * np.eye(S) + 0.25 * rng.standard_normal((S, S)) / np.sqrt(S)
            else:
                vec(f"{p}norm{q}b", D)
        x = p + "mix."
        if l["type"] == "latent_attention":
            H, size = m["heads"], m["dim"] + m["rot_dim"]
            mat(x + "dq", m["q_rank"], D)
            vec(x + "dq.norm", m["q_rank"])
            mat(x + "uq", H * size, m["q_rank"], 1.5)
            mat(x + "dkv", m["kv_rank"] + m["rot_dim"], D)
            vec(x + "dkv.norm", m["kv_rank"])
            mat(x + "uk", H * m["dim"], m["kv_rank"], 1.5)
            mat(x + "uv", H * m["vdim"], m["kv_rank"])
            if sinks:
                vec(x + "sink", H, 0.5, 1.0)
            mat(x + "o", D, H * m["vdim"], 1.5)
        elif l["type"] == "mamba2":
            H, inner, C = m["heads"], m["heads"] * m["vdim"], m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"]
            mat(x + "in", inner + C + H, D)
            W[x + "conv"] = rng.standard_normal((C, m["conv"])) * 0.6
            vec(x + "conv.b", C, 0.2, 0.3)
            vec(x + "dt_bias", H, -1.5, 0.7)
            vec(x + "A_log", H, -0.5, 0.7)
            vec(x + "D", H, 0.8, 0.4)
            vec(x + "norm", inner)
            mat(x + "o", D, inner)
        if l["mlp"] and l["mlp"]["kind"] == "dense":
            mat(p + "mlp.gate", l["mlp"]["ff"], D, 1.5)
            mat(p + "mlp.up", l["mlp"]["ff"], D, 1.5)
            mat(p + "mlp.down", D, l["mlp"]["ff"])
    norm("final.norm")
    if not tied:
        mat("head", cfg["vocab"], D, 2.0)
    return {k: bb.to_bf16(v).reshape(np.shape(v)) for k, v in W.items()}


def specs(cfg, W):
    """the layers as lv_block_spec; flags and activation follow what weights and configuration hold"""
    lva = importlib.import_module("llama-vulkan_amd")
    out = []
    for i, l in enumerate(cfg["layers"]):
        m, x = l["mixer"], f"l{i}.mix."
        b = lva.BlockSpec()
        if l["type"] == "parallel":
            b = bb.specs({"layers": [l]}, {k.replace(f"l{i}.", "l0."): v for k, v in W.items()})[0]
        elif l["type"] == "latent_attention":
            b.latent = lva.LatentSpec(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["q_rank"], m["kv_rank"], m["scale"], m["rot"]["dims"], m["rot"]["base"],
                                      lva.ATTN_SINK if x + "sink" in W else 0)
        else:
            b.ssm = lva.SsmSpec(m["heads"], m["groups"], m["state"], m["vdim"], m["conv"], m["norm_groups"])
        if l["mlp"] and l["mlp"]["kind"] == "dense":
            b.dense = lva.DenseSpec(l["mlp"]["ff"], lva.ACT_SILU if l["mlp"].get("act") == "silu" else lva.ACT_RELU)
        out.append(b)
    return out


def upload(ctx, cfg, W, compute):
    """BlockModel straight through the C-ABI"""
    lva = importlib.import_module("llama-vulkan_amd")
    g, loop = cfg["embedding"].get("bigram"), cfg.get("loop")
    wide = dict(norm=lva.NORM_TANH if "final.norm.alpha" in W else lva.NORM_RMS, streams=cfg["streams"], tied_head=int("head" not in W), embed_scale=cfg["embedding"]["scale"])
    if g:
        wide.update(bigram_buckets=g["buckets"], bigram_prev=g["mul_prev"], bigram_cur=g["mul_cur"])
    if loop:
        wide.update(loop_start=loop["start"], loop_stop=loop["stop"], loop_times=loop["times"])
    return bb.upload(ctx, cfg, W, compute, blocks=specs(cfg, W), **wide)
