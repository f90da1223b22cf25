"""Small random Gamilorn models for the tests: configurations, weights, checkpoint files (not collected by pytest)."""
import importlib
import json
import os
import struct

import numpy as np


def bits_and_values(x):
    """bf16 bits of x and what they stand for, in float64."""
    synth = importlib.import_module("turbo_lossless_amd.synth")
    b = synth.f32_to_bf16_bits(np.asarray(x, np.float32)).reshape(np.shape(x))
    return b, synth.bf16_bits_to_f32(b).reshape(b.shape).astype(np.float64)


def layer(heads=4, kv_heads=2, dim=32, vdim=32, window=20, keep=3, d_heads=2, d_dim=32, ff=96, scale=None, ls=0.9, rs=1.3):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5,
            "mask": {"size": window, "keep_first": keep}}
    return {"type": "parallel", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"left": left, "right": {"heads": d_heads, "dim": d_dim}, "left_scale": ls, "right_scale": rs}}


def config(layers, vocab=97, width=64, positions=512, eps=1e-5, cap=20.0):
    return {"architecture": "Gamilorn", "layers": layers, "vocab": vocab, "width": width, "max_positions": positions,
            "norm": {"eps": eps}, "logit_softcap": cap}


def tensors(cfg, rank, seed):
    """{name: float array before rounding} of every tensor of the checkpoint."""
    rng = np.random.default_rng(seed)
    n = cfg["width"]
    mat = lambda m, k, gain=1.0: rng.standard_normal((m, k)) * gain / np.sqrt(k)
    vec = lambda m, mean=0.0, dev=0.3: mean + dev * rng.standard_normal(m)
    t = {"embed": rng.standard_normal((cfg["vocab"], n)), "pos": 0.3 * rng.standard_normal((cfg["max_positions"], n)),
         "final.norm": vec(n), "head": mat(cfg["vocab"], n, 4.0)}
    for i, L in enumerate(cfg["layers"]):
        a, b, p = L["mixer"]["left"], L["mixer"]["right"], "l%d." % i
        d = b["heads"] * b["dim"]
        t[p + "norm1"] = vec(n)
        for name, m in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
            t[p + "mix.left." + name] = mat(m, n, 1.5 if name != "v" else 1.0)
            t[p + "mix.left.%s.b" % name] = vec(m)
        t[p + "mix.left.pb"] = vec(a["heads"], -2.5)
        t[p + "mix.left.o"] = mat(n, a["heads"] * a["vdim"], 0.7)
        for name in "rkvga":
            t[p + "mix.right." + name] = mat(d, n)
        t[p + "mix.right.a.b"] = vec(d, 0.0, 1.5)
        t[p + "mix.right.w1"] = mat(rank, n)
        t[p + "mix.right.w2"] = mat(d, rank)
        t[p + "mix.right.w0"] = vec(d, -3.0, 3.0)
        t[p + "mix.right.norm"] = vec(d, 1.0)
        t[p + "mix.right.o"] = mat(n, d, 0.7)
        if L["mlp"]:
            ff = L["mlp"]["ff"]
            t[p + "norm2"] = vec(n)
            t[p + "mlp.up"] = mat(ff, n)
            t[p + "mlp.down"] = mat(n, ff, 0.5)
            t[p + "mlp.act"] = vec(2, 0.6, 0.4)
    return t


def write_checkpoint(path, cfg, t):
    """config.json + model.safetensors; returns the tensors as stored (float64) for the oracle."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blobs, at, values = {}, [], 0, {}
    for name, x in t.items():
        b, values[name] = bits_and_values(x)
        header[name] = {"dtype": "BF16", "shape": list(b.shape), "data_offsets": [at, at + b.nbytes]}
        blobs.append(b.tobytes())
        at += b.nbytes
    h = json.dumps(header).encode()
    h += b" " * (-len(h) % 8)
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + b"".join(blobs))
    return values


def error(got, want):
    """RMS of the difference over the RMS of what is wanted, the worst row."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    return float((np.sqrt(np.mean((got - want) ** 2, axis=-1)) / np.sqrt(np.mean(want ** 2))).max())
