"""Small random Davasun models for the tests: configurations, weights, checkpoint files (not collected by pytest)."""
import numpy as np

from gamilorn_util import bits_and_values, error, write_checkpoint  # noqa: F401  (shared with the tests that import this)


def mlstm(heads=2, dim=24, vdim=40, cap=9.0, ff=0, limit=1.5):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": dense(ff, limit)}


def latent(heads=3, dim=32, rot=16, vdim=24, rank=64, base=500.0, scale=None, ff=80, limit=1.5):
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": scale or 1.5 * (dim + rot) ** -0.5,
             "rot": {"dims": rot, "base": base}}
    return {"type": "latent_attention", "mixer": mixer, "mlp": dense(ff, limit)}


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit} if ff else None


def config(layers, vocab=97, width=64, eps=1e-5, logit_scale=3.0, loop=None):
    return {"architecture": "Davasun", "layers": layers, "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale,
            "loop": {"start": loop[0], "stop": loop[1], "times": loop[2]} if loop else None}


def tensors(cfg, seed):
    """{name: float array before rounding} of every tensor of the checkpoint."""
    rng = np.random.default_rng(seed)
    n = cfg["width"]
    mat = lambda m, k, gain=1.0: rng.standard_normal((m, k)) * gain / np.sqrt(k)
    vec = lambda m, mean=0.0, dev=0.3: mean + dev * rng.standard_normal(m)
    gain = lambda: np.array(rng.uniform(0.6, 1.5))
    t = {"embed": rng.standard_normal((cfg["vocab"], n)), "embed.norm": gain(), "final.norm": gain(), "head": mat(cfg["vocab"], n)}
    for i, L in enumerate(cfg["layers"]):
        c, p = L["mixer"], "l%d." % i
        H, hv = c["heads"], c["heads"] * c["vdim"]
        t[p + "norm1"], t[p + "norm1b"] = gain(), gain()
        if L["type"] == "mlstm":
            # (keys that resemble their queries: the normaliser seldom cancels, so rounding stays small)
            t[p + "mix.q"] = mat(H * c["dim"], n, 1.5)
            t[p + "mix.k"] = 0.8 * t[p + "mix.q"] + mat(H * c["dim"], n, 0.9)
            for name in "vg":
                t[p + "mix." + name] = mat(hv, n)
            t[p + "mix.norm"] = vec(hv, 1.0)
            t[p + "mix.i"], t[p + "mix.i.b"] = mat(H, n, 2.0), vec(H, -1.0, 1.5)
            t[p + "mix.f"], t[p + "mix.f.b"] = mat(H, n, 2.0), vec(H, 3.0, 1.5)
        else:
            d, r, R = c["dim"], c["rot_dim"], c["kv_rank"]
            t[p + "mix.q"], t[p + "mix.g"] = mat(H * (d + r), n, 1.5), mat(H, n)
            t[p + "mix.dkv"], t[p + "mix.dkv.norm"] = mat(R + r, n, 1.2), vec(R, 1.0)
            t[p + "mix.uk"], t[p + "mix.uv"] = mat(H * d, R), mat(hv, R)
        t[p + "mix.o"] = mat(n, hv)
        if L["mlp"]:
            ff = L["mlp"]["ff"]
            t[p + "norm2"], t[p + "norm2b"] = gain(), gain()
            t[p + "mlp.gate"], t[p + "mlp.up"], t[p + "mlp.down"] = mat(ff, n, 1.5), mat(ff, n, 1.5), mat(n, ff)
    return t
