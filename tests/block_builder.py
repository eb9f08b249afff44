"""Small random block models for the tests: configurations, weights (bf16-exact), model folders, and direct uploads through the
C-ABI for layer forms that no design uses."""
import importlib
import json
import os
import struct

import numpy as np


def attn(heads=3, kv_heads=1, dim=20, chunk=12, rot=None, scale=None, base=1000.0):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "mask": {"size": chunk},
            "rot": {"dims": dim if rot is None else rot, "base": base}, "scale": dim ** -0.5 if scale is None else scale}


def delta(heads=4, kv_heads=2, dim=12, vdim=20, conv=3):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def layer(left=None, right=None, experts=5, top=2, ff=24, left_scale=0.7, right_scale=1.1, without=()):
    return {"type": "parallel",
            "mixer": {"left": None if "left" in without else left or attn(), "right": None if "right" in without else right or delta(),
                      "left_scale": left_scale, "right_scale": right_scale},
            "mlp": {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}} if experts else None}


def config(vocab=53, width=40, layers=None, eps=1e-5):
    return {"architecture": "Somesun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers or [layer(), layer(experts=0), layer(top=1)]}


def to_bf16(a):
    """nearest bf16 bits (ties to even) of a float array"""
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def from_bf16(b):
    return (b.astype(np.uint32) << 16).view(np.float32).astype(np.float64)


def weights(cfg, seed, rank_a=7, rank_g=9, values=False, norms=True, sinks=True):
    """name -> bf16 bits.  values: attention layers get a value projection of their own; norms, sinks: whether they have those"""
    rng = np.random.default_rng(seed)
    D, W = cfg["width"], {}

    def mat(name, rows, cols, gain=1.0):
        W[name] = rng.standard_normal((rows, cols)) * gain / np.sqrt(cols)

    def vec(name, n, mean=1.0, spread=0.2):
        W[name] = mean + spread * rng.standard_normal(n)

    W["embed"] = rng.standard_normal((cfg["vocab"], D))
    for i, l in enumerate(cfg["layers"]):
        p = f"l{i}."
        for n in ["norm1", "norm1b"] + (["norm2", "norm2b"] if l["mlp"] else []):
            vec(p + n, D)
        a, d = l["mixer"]["left"], l["mixer"]["right"]
        if a:
            pa = p + "mix.left."
            mat(pa + "q", a["heads"] * a["dim"], D)
            mat(pa + "k", a["kv_heads"] * a["dim"], D)
            if values:
                mat(pa + "v", a["kv_heads"] * a["vdim"], D)
            if norms:
                vec(pa + "q.norm", a["heads"] * a["dim"])
                vec(pa + "k.norm", a["kv_heads"] * a["dim"])
            if sinks:
                vec(pa + "sink", a["heads"], 0.5, 1.0)
            mat(pa + "o", D, a["heads"] * a["vdim"])
        if d:
            pd = p + "mix.right."
            nq, nv = d["kv_heads"] * d["dim"], d["heads"] * d["vdim"]
            for n, rows in (("q", nq), ("k", nq), ("v", nv)):
                mat(pd + n, rows, D)
                W[pd + n + ".conv"] = rng.standard_normal((rows, d["conv"])) * 0.6
            mat(pd + "b", d["heads"], D)
            mat(pd + "a1", rank_a, D)
            mat(pd + "a2", d["heads"] * d["dim"], rank_a)
            mat(pd + "g1", rank_g, D)
            mat(pd + "g2", nv, rank_g)
            vec(pd + "A_log", d["heads"], -1.0, 0.7)
            vec(pd + "dt_bias", d["heads"] * d["dim"], -1.5, 0.7)
            vec(pd + "norm", d["vdim"])
            mat(pd + "o", D, nv)
        if l["mlp"]:
            mat(p + "mlp.router", l["mlp"]["router"]["experts"], D, 1.5)
            for e in range(l["mlp"]["router"]["experts"]):
                for n in ("gate", "up"):
                    mat(f"{p}mlp.e{e}.{n}", l["mlp"]["expert"]["ff"], D, 1.5)
                mat(f"{p}mlp.e{e}.down", D, l["mlp"]["expert"]["ff"])
    vec("final.norm", D)
    mat("head", cfg["vocab"], D, 2.0)
    return {k: to_bf16(v) for k, v in W.items()}


def as_float(W):
    return {k: from_bf16(v) for k, v in W.items()}


def write_folder(path, cfg, seed=0, W=None):
    """config.json and model.safetensors; returns the weights"""
    os.makedirs(path, exist_ok=True)
    W = W or weights(cfg, seed)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, off = {}, 0
    for k, v in W.items():
        head[k] = {"dtype": "BF16", "shape": list(v.shape), "data_offsets": [off, off + v.nbytes]}
        off += v.nbytes
    text = json.dumps(head).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text)
        for v in W.values():
            f.write(v.tobytes())
    return W


def specs(cfg, W):
    """the layers as lv_block_spec, flags following what the weights hold"""
    lva = importlib.import_module("llama-vulkan_amd")
    out = []
    for i, l in enumerate(cfg["layers"]):
        b = lva.BlockSpec()
        m, p = l["mixer"], f"l{i}.mix.left."
        b.attn_scale, b.delta_scale = m["left_scale"], m["right_scale"]
        if m["left"]:
            a = m["left"]
            flags = (lva.ATTN_NORM_FULL if p + "q.norm" in W else 0) | (0 if p + "v" in W else lva.ATTN_KEYS_AS_VALUES) | (lva.ATTN_SINK if p + "sink" in W else 0)
            b.attn = lva.AttnSpec(a["heads"], a["kv_heads"], a["dim"], a["vdim"], a["scale"], a["mask"]["size"], a["rot"]["dims"], a["rot"]["base"], flags)
        if m["right"]:
            d = m["right"]
            b.delta = lva.DeltaSpec(d["heads"], d["kv_heads"], d["dim"], d["vdim"], d["conv"])
        if l["mlp"]:
            b.moe = lva.MoeSpec(l["mlp"]["router"]["experts"], l["mlp"]["router"]["top"], l["mlp"]["expert"]["ff"])
        out.append(b)
    return out


def upload(ctx, cfg, W, compute, blocks=None, **model_wide):
    """BlockModel straight through the C-ABI"""
    lva = importlib.import_module("llama-vulkan_amd")
    base = np.concatenate([v.reshape(-1) for v in W.values()]).view(np.uint8)
    table, off = [], 0
    for k, v in W.items():
        table.append((k, lva.LV_BF16, off, v.shape[0] if v.ndim else 1, v.shape[1] if v.ndim == 2 else 1, v.nbytes))
        off += v.nbytes
    return lva.BlockModel(ctx, base, table, blocks or specs(cfg, W), cfg["vocab"], cfg["width"], cfg["norm"]["eps"], compute, **model_wide)
