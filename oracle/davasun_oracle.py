"""Plain restatement of the Davasun decoder in float64 numpy, one function per mechanism.  Slow on purpose: every recurrent
step is taken one by one, every query looks at its keys on its own, keys and values are formed per head.  Shares no code
with the product path; imported by tests only.

A model is a dict: the configuration as config.json spells it, and tensors {name: float64 array} under the checkpoint's
names.  Linear weights are [out, in].
"""
from __future__ import annotations

import numpy as np


def sigmoid(x):
    x = np.asarray(x, np.float64)
    e = np.exp(-np.abs(x))
    return np.where(x >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def log_sigmoid(x):
    return -np.logaddexp(0.0, -np.asarray(x, np.float64))


def soft_cap(x, cap):
    return cap * np.tanh(x / cap)


def rms(x, eps):
    """x over its root mean square along the last axis, eps under the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm_one_gain(x, g, eps):
    """RMS norm with a single gain for all coordinates."""
    return rms(x, eps) * float(g)


def norm_plain(x, w, eps):
    return rms(x, eps) * w


# ---- matrix memory ---------------------------------------------------------------------------------------------------
def memory_step(S, n, m, q, k, v, i, f):
    """One token of one head.  S [d, e], n [d], m the running maximum; i, f the log gates.  Returns (S, n, m, output)."""
    new = max(f + m, i)
    keep, enter = np.exp(f + m - new), np.exp(i - new)
    S = keep * S + enter * np.outer(k, v)
    n = keep * n + enter * k
    return S, n, new, (S.T @ q) / (max(abs(n @ q), np.exp(-new)) + 1e-6)


def memory_scan(q, k, v, i, f, S, n, m):
    """q, k [T, H, d], v [T, H, e], i, f [T, H]; state S [H, d, e], n [H, d], m [H].  Returns (o [T, H, e], S, n, m)."""
    T, H, _ = q.shape
    S, n, m = S.copy(), n.copy(), m.copy()
    o = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        for h in range(H):
            S[h], n[h], m[h], o[t, h] = memory_step(S[h], n[h], m[h], q[t, h], k[t, h], v[t, h], i[t, h], f[t, h])
    return o, S, n, m


def memory_gates(h, wi, bi, wf, bf, cap):
    return soft_cap(h @ wi.T + bi, cap), log_sigmoid(soft_cap(h @ wf.T + bf, cap))


def gated_heads(o, w, gate, eps):
    """Heads over their own RMS, concatenated, times a plain weight and a sigmoid gate."""
    return rms(o, eps).reshape(o.shape[0], -1) * w * sigmoid(gate)


def mixer_mlstm(T_, pre, c, h, st, pos, eps):
    n, H, d, e = h.shape[0], c["heads"], c["dim"], c["vdim"]
    w = lambda name: T_[pre + name]
    q = (h @ w("q").T).reshape(n, H, d) / np.sqrt(d)
    k = (h @ w("k").T).reshape(n, H, d)
    v = (h @ w("v").T).reshape(n, H, e)
    i, f = memory_gates(h, w("i"), w("i.b"), w("f"), w("f.b"), c["gate_cap"])
    o, st["S"], st["n"], st["m"] = memory_scan(q, k, v, i, f, st["S"], st["n"], st["m"])
    return gated_heads(o, w("norm"), h @ w("g").T, eps) @ w("o").T


# ---- latent attention ------------------------------------------------------------------------------------------------
def rotate_half(x, positions, base):
    """Coordinate i of the last axis and coordinate i + size / 2 are a pair, turned by position * base^(-2 i / size)."""
    half = x.shape[-1] // 2
    a = np.asarray(positions, np.float64)[:, None] * float(base) ** (-2.0 * np.arange(half) / x.shape[-1])
    a = a.reshape(a.shape[0], *([1] * (x.ndim - 2)), half)
    u, v = x[..., :half], x[..., half:]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a)], axis=-1)


def causal_attention(q, k, v, scale, first):
    """q [T, H, d] at positions first ...; k [N, H, d], v [N, H, e] at positions 0 ... N - 1; softmax.  [T, H, e]."""
    T, H, _ = q.shape
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        for h in range(H):
            s = k[:first + t + 1, h] @ q[t, h] * scale
            p = np.exp(s - s.max())
            out[t, h] = (p / p.sum()) @ v[:first + t + 1, h]
    return out


def mixer_latent(T_, pre, c, h, st, pos, eps):
    n, H, d, r, e, R = h.shape[0], c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
    w = lambda name: T_[pre + name]
    at = np.arange(pos, pos + n)
    q = (h @ w("q").T).reshape(n, H, d + r)
    q = np.concatenate([q[..., :d], rotate_half(q[..., d:], at, c["rot"]["base"])], axis=-1)
    x = h @ w("dkv").T
    st["c"] = np.concatenate([st["c"], norm_plain(x[:, :R], w("dkv.norm"), eps)])
    st["r"] = np.concatenate([st["r"], rotate_half(x[:, R:], at, c["rot"]["base"])])
    N = len(st["c"])
    k = (st["c"] @ w("uk").T).reshape(N, H, d)
    k = np.concatenate([k, np.broadcast_to(st["r"][:, None], (N, H, r))], axis=-1)
    v = (st["c"] @ w("uv").T).reshape(N, H, e)
    o = causal_attention(q, k, v, c["scale"], pos) * sigmoid(h @ w("g").T)[:, :, None]
    return o.reshape(n, H * e) @ w("o").T


# ---- feed-forward ----------------------------------------------------------------------------------------------------
def clamped_glu(gate, up, limit):
    g, u = np.minimum(gate, limit), np.clip(up, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


# ---- the whole -------------------------------------------------------------------------------------------------------
def order(cfg):
    """Layer indices in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


class State:
    """What one sequence leaves behind, per layer run."""

    def __init__(self, cfg):
        self.pos, self.runs = 0, []
        for i in order(cfg):
            c = cfg["layers"][i]["mixer"]
            if cfg["layers"][i]["type"] == "mlstm":
                self.runs.append(dict(S=np.zeros((c["heads"], c["dim"], c["vdim"])), n=np.zeros((c["heads"], c["dim"])),
                                      m=np.zeros(c["heads"])))
            else:
                self.runs.append(dict(c=np.zeros((0, c["kv_rank"])), r=np.zeros((0, c["rot_dim"]))))


MIXERS = {"mlstm": mixer_mlstm, "latent_attention": mixer_latent}


def forward(cfg, T_, tokens, state=None, want_layers=False):
    """Runs `tokens` from where `state` stands; returns logits [T, vocab] (and the residual after every layer run)."""
    state = state or State(cfg)
    eps = cfg["norm"]["eps"]
    x = norm_one_gain(T_["embed"][np.asarray(tokens)], T_["embed.norm"], eps)
    trail = []
    for st, i in zip(state.runs, order(cfg)):
        L, p = cfg["layers"][i], "l%d." % i
        y = MIXERS[L["type"]](T_, p + "mix.", L["mixer"], norm_one_gain(x, T_[p + "norm1"], eps), st, state.pos, eps)
        x = x + norm_one_gain(y, T_[p + "norm1b"], eps)
        if L.get("mlp"):
            h = norm_one_gain(x, T_[p + "norm2"], eps)
            y = clamped_glu(h @ T_[p + "mlp.gate"].T, h @ T_[p + "mlp.up"].T, L["mlp"]["limit"]) @ T_[p + "mlp.down"].T
            x = x + norm_one_gain(y, T_[p + "norm2b"], eps)
        trail.append(x)
    state.pos += len(tokens)
    logits = norm_one_gain(x, T_["final.norm"], eps) @ T_["head"].T * cfg["logit_scale"]
    return (logits, np.stack(trail)) if want_layers else logits
