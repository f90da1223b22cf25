"""GPU: every mechanism of the Davasun layers through the C ABI, alone, against the float64 oracle: matrix memory (token step,
exact scan, chunks on the matrix cores), latent attention (matrix-core and general forms, either precision), norms around
sublayers, the normed embedding, the clamped gated unit and the fused forms of the products."""
import ctypes as C

import numpy as np
import pytest
import torch

from davasun_util import bits_and_values
from gpu_util import dev, rel_err
from oracle import davasun_oracle as do

pytestmark = pytest.mark.gpu


def up(x, dtype=torch.float32):
    return torch.from_numpy(np.ascontiguousarray(x)).to(dev()).to(dtype)


def bf16(x):
    return bits_and_values(x)[1]


def host(x):
    return x.float().cpu().numpy().astype(np.float64)


def off(got, want, every):
    """Largest difference against the largest value there is anywhere."""
    return float(np.abs(got - want).max() / np.abs(every).max())


def row_table(t12, pos, slots):
    n = len(pos)
    rows = (t12.Row * n)(*[t12.Row(int(p), int(s)) for p, s in zip(pos, slots)])
    d = torch.empty(2 * n, dtype=torch.int32, device=dev())
    t12.check(t12.lib.t12_rows_list(d.data_ptr(), rows, n, t12.current_stream()))
    return d


# ------------------------------------------------------------------------------------------------- matrix memory
class Memory:
    """Regions of a matrix memory, fed with projections row by row or run by run."""

    def __init__(self, t12, heads, dim, vdim, regions=1, cap=10.0, rows=512, seed=0):
        self.t12, self.H, self.D, self.V, self.cap = t12, heads, dim, vdim, cap
        self.norm = 1 + 0.3 * np.random.default_rng(seed).standard_normal(heads * vdim)
        self.norm_d = up(self.norm)
        m = self.m = t12.MatrixMemory()
        m.heads, m.dim, m.vdim, m.q_scale, m.gate_cap, m.den_eps, m.out_eps = heads, dim, vdim, dim ** -0.5, cap, 1e-6, 1e-5
        m.norm_w = self.norm_d.data_ptr()
        self.off = {}
        at = 0
        for name, n in (("q", heads * dim), ("k", heads * dim), ("v", heads * vdim), ("g", heads * vdim), ("i", heads), ("f", heads)):
            setattr(m, name + "_off", at)
            self.off[name] = slice(at, at + n)
            at += n
        self.ld = (at + 3) // 4 * 4 if dim % 4 == 0 else at + 3
        t12.check(t12.lib.t12_memory_plan(C.byref(m), rows))
        # what a region holds before position 0 must not matter, not even when it is no number
        self.state = torch.full((regions * 2 * m.state_elems,), float("nan"), device=dev())
        m.state = self.state.data_ptr()
        self.work = torch.empty(m.work_floats, device=dev())
        self.parity = [0] * regions

    def inputs(self, n, seed, gate=2.0):
        rng = np.random.default_rng(seed)
        x = rng.standard_normal((n, self.ld))
        x[:, self.off["i"]] = gate * x[:, self.off["i"]] - 1
        x[:, self.off["f"]] = gate * x[:, self.off["f"]] + 3
        return bf16(x)

    def feed(self, x, pos, region, exact=False, fp32=True):
        n, t12 = len(x), self.t12
        run = not isinstance(region, (list, tuple))
        regions = [region] * n if run else region
        dr = row_table(t12, pos, [2 * g + self.parity[g] for g in regions])
        xi, bi = up(x - 0.25), up(np.full(self.ld, 0.25))               # a bias the kernels add back
        out = torch.zeros((n, self.H * self.V), dtype=torch.float32 if fp32 else torch.bfloat16, device=dev())
        t12.check(t12.lib.t12_matrix_memory(C.byref(self.m), xi.data_ptr(), bi.data_ptr(), self.ld, dr.data_ptr(), n, int(run), int(exact),
                                            self.work.data_ptr(), out.data_ptr(), int(fp32), self.H * self.V, t12.current_stream()))
        torch.cuda.synchronize()
        for g in set(regions):
            self.parity[g] ^= 1
        return host(out)

    def oracle(self, x):
        n, H, D, V = len(x), self.H, self.D, self.V
        g = {k: x[:, s] for k, s in self.off.items()}
        i, f = do.soft_cap(g["i"], self.cap), do.log_sigmoid(do.soft_cap(g["f"], self.cap))
        o, *_ = do.memory_scan(g["q"].reshape(n, H, D) / np.sqrt(D), g["k"].reshape(n, H, D), g["v"].reshape(n, H, V), i, f,
                               np.zeros((H, D, V)), np.zeros((H, D)), np.zeros(H))
        return do.gated_heads(o, self.norm, g["g"], 1e-5)


MEMORY = [(2, 24, 40), (3, 20, 12), (1, 64, 64), (2, 128, 15), (2, 160, 96), (1, 256, 131), (1, 300, 33), (1, 512, 48), (5, 8, 200), (1, 1, 1)]


@pytest.mark.parametrize("heads, dim, vdim", MEMORY)
@pytest.mark.parametrize("exact", [False, True])
def test_memory_in_any_portions(t12, heads, dim, vdim, exact):
    M = Memory(t12, heads, dim, vdim)
    n = 150
    x = M.inputs(n, dim + vdim)
    want = M.oracle(x)
    for cuts in ([150], [64, 64, 22], [63, 2, 65, 1, 19], [2] * 75):
        at = 0
        for c in cuts:
            got = M.feed(x[at:at + c], range(at, at + c), 0, exact)
            assert rel_err(got, want[at:at + c]) < 1e-4, (cuts[:5], at)
            at += c


@pytest.mark.parametrize("heads, dim, vdim", MEMORY)
def test_memory_token_by_token(t12, heads, dim, vdim):
    M = Memory(t12, heads, dim, vdim)
    x = M.inputs(80, 7 * dim + vdim)
    want = M.oracle(x)
    got = np.concatenate([M.feed(x[i:i + 1], [i], [0]) for i in range(80)])
    assert rel_err(got, want) < 1e-4
    got = np.concatenate([M.feed(x[:37], range(37), 0)] + [M.feed(x[i:i + 1], [i], [0], fp32=False) for i in range(37, 80)])
    assert rel_err(got, want) < 5e-3


@pytest.mark.parametrize("exact", [False, True])
@pytest.mark.parametrize("gate, cap", [(30.0, 14.0), (0.1, 3.0), (8.0, 40.0)])
def test_memory_gates_at_their_limits(t12, gate, cap, exact):
    """Gates pressed against their cap: tokens that wipe the past or hardly enter, a maximum that jumps."""
    M = Memory(t12, 3, 32, 48, cap=cap)
    x = M.inputs(200, 3, gate)
    want = M.oracle(x)
    got = np.concatenate([M.feed(x[:140], range(140), 0, exact)] + [M.feed(x[i:i + 1], [i], [0]) for i in range(140, 200)])
    # (where the normaliser nearly cancels, its rounding shows: rows are judged by their own size)
    err = np.sqrt(np.mean((got - want) ** 2, 1) / np.mean(want ** 2, 1))
    assert np.isfinite(got).all() and np.median(err) < 1e-5 and err.max() < 2e-2


@pytest.mark.parametrize("exact", [False, True])
@pytest.mark.parametrize("place", [0, 1, 62, 63, 64, 65, 127, 128, 190])
def test_one_token_far_back_is_read_out(t12, place, exact):
    """All input gates are shut but that of one token; queries point at its key: its value must come back at any distance, in a
    run and decoded, and nothing of it before."""
    M = Memory(t12, 2, 32, 24)
    n = 260
    x = M.inputs(n, place)
    x[:, M.off["i"]], x[:, M.off["f"]] = -9.5, 30.0
    x[place, M.off["i"]] = 6.0
    x[:, M.off["q"]] = bf16(4 * x[place, M.off["k"]])
    want = M.oracle(x)
    shut = x.copy()
    shut[place, M.off["i"]] = -9.5
    plain = M.oracle(shut)
    assert rel_err(plain[place:], want[place:]) > 0.1                  # (the token shows)
    got = np.concatenate([M.feed(x[:100], range(100), 0, exact), M.feed(x[100:230], range(100, 230), 0, exact)] +
                         [M.feed(x[i:i + 1], [i], [0]) for i in range(230, n)])
    assert rel_err(got, want) < 1e-4


def test_memory_lasts_and_restarts_at_zero(t12):
    M = Memory(t12, 2, 64, 80)
    x = M.inputs(900, 1)
    x[:, M.off["f"]] = 30.0                                            # nothing is forgotten
    want = M.oracle(x)
    got = np.concatenate([M.feed(x[:512], range(512), 0), M.feed(x[512:800], range(512, 800), 0)] +
                         [M.feed(x[i:i + 1], [i], [0]) for i in range(800, 900)])
    assert rel_err(got, want) < 2e-4
    assert rel_err(M.feed(x[5:30], range(25), 0), M.oracle(x[5:30])) < 1e-4
    assert rel_err(M.feed(x[7:8], [0], [0]), M.oracle(x[7:8])) < 1e-4


def test_memory_step_taken_back(t12):
    M = Memory(t12, 2, 32, 16)
    x = M.inputs(12, 2)
    M.feed(x[:10], range(10), 0)
    M.feed(x[11:12], [10], [0])                                        # a token that is then taken back
    M.parity[0] ^= 1
    assert rel_err(M.feed(x[10:11], [10], [0]), M.oracle(x[:11])[10:]) < 1e-4


@pytest.mark.parametrize("B, heads, dim, vdim", [(3, 2, 32, 40), (70, 4, 64, 128), (40, 3, 256, 300)])
def test_memory_rows_of_their_own(t12, B, heads, dim, vdim):
    """A batch of unequal sequences decoded together (both shapes of the step's launch), one of them at its first token."""
    M = Memory(t12, heads, dim, vdim, regions=B)
    rng = np.random.default_rng(B)
    lens = [0] + [int(rng.integers(1, 20)) for _ in range(B - 1)]
    seqs = [M.inputs(n + 3, 50 + b) for b, n in enumerate(lens)]
    for b in range(B):
        if lens[b]:
            M.feed(seqs[b][:lens[b]], range(lens[b]), b)
    want = [M.oracle(s) for s in seqs]
    for s in range(3):
        got = M.feed(np.stack([seqs[b][lens[b] + s] for b in range(B)]), [n + s for n in lens], list(range(B)))
        for b in range(B):
            assert rel_err(got[b], want[b][lens[b] + s]) < 1e-4, (b, s)


# ----------------------------------------------------------------------------------------------- latent attention
def packed(t12, oracle, w):
    """Split-12 tensor of w [M, K]; returns (device tensor, the values it stands for)."""
    bits, values = bits_and_values(w)
    return t12.DeviceTensor12.from_packed(oracle.pack(bits), dev()), values


class Latent:
    """Regions of a latent cache, fed with projections row by row or run by run."""

    def __init__(self, t12, oracle, heads, dim, rot, vdim, rank, fp32=False, regions=1, rows=256, positions=4096, scale=None, uk=None, uv=None,
                 base=300.0, seed=0):
        self.t12, self.H, self.d, self.r, self.e, self.R, self.fp32, self.base = t12, heads, dim, rot, vdim, rank, fp32, base
        self.scale = scale or 1.2 / np.sqrt(dim + rot)
        rng = np.random.default_rng(seed)
        uk = rng.standard_normal((heads * dim, rank)) / np.sqrt(rank) if uk is None else uk
        uv = rng.standard_normal((heads * vdim, rank)) / np.sqrt(rank) if uv is None else uv
        far = rng.random(uk.shape) < 3e-3                              # weights outside the packed range: escapes
        kt, _ = packed(t12, oracle, np.where(far, 40.0 * uk, uk).reshape(heads, dim, rank).transpose(0, 2, 1).reshape(heads * rank, dim))
        self.uk = bf16(np.where(far, 40.0 * uk, uk))
        vt, self.uv = packed(t12, oracle, np.where(rng.random(uv.shape) < 3e-3, 40.0 * uv, uv))
        self.norm = bf16(1 + 0.3 * rng.standard_normal(rank))
        self.norm_d, self.freqs = up(self.norm), up(base ** (-2.0 * np.arange(rot // 2) / rot))
        self.keep = (kt, vt)
        self.segs = [kt.segment(None), vt.segment(None)]
        a = self.a = t12.LatentAttn()
        a.heads, a.dim, a.rot_dim, a.vdim, a.rank, a.scale, a.eps, a.elem_bytes = heads, dim, rot, vdim, rank, self.scale, 1e-5, 4 if fp32 else 2
        a.k_up, a.v_up = C.pointer(self.segs[0]), C.pointer(self.segs[1])
        a.norm_w, a.freqs = self.norm_d.data_ptr(), self.freqs.data_ptr()
        a.q_off, a.c_off, a.g_off = 0, heads * (dim + rot), heads * (dim + rot) + rank + rot
        self.ld = a.g_off + heads
        t12.check(t12.lib.t12_latent_plan(C.byref(a), positions, rows))
        self.cache = torch.zeros(regions * a.cache_elems, dtype=torch.float32 if fp32 else torch.int16, device=dev())
        a.cache = self.cache.data_ptr()
        self.work = torch.empty(a.work_floats, device=dev())

    def inputs(self, n, seed):
        return bf16(np.random.default_rng(seed).standard_normal((n, self.ld)))

    def feed(self, x, pos, region):
        n, t12 = len(x), self.t12
        run = not isinstance(region, (list, tuple))
        dr = row_table(t12, pos, [2 * g for g in ([region] * n if run else region)])
        xi = up(x)
        out = torch.zeros((n, self.H * self.e), dtype=torch.float32 if self.fp32 else torch.bfloat16, device=dev())
        t12.check(t12.lib.t12_latent_attention(C.byref(self.a), xi.data_ptr(), self.ld, dr.data_ptr(), n, int(run), int(max(pos)),
                                               self.work.data_ptr(), out.data_ptr(), int(self.fp32), self.H * self.e, t12.current_stream()))
        torch.cuda.synchronize()
        return host(out)

    def oracle(self, x, past=None, first=0):
        """Rows x at positions first ...; past: the rows before them."""
        every = x if past is None else np.concatenate([past, x])
        start = first - (0 if past is None else len(past))
        n, H, d, r, e, R = len(every), self.H, self.d, self.r, self.e, self.R
        at = np.arange(start, start + n)
        q = every[:, :H * (d + r)].reshape(n, H, d + r)
        q = np.concatenate([q[..., :d], do.rotate_half(q[..., d:], at, self.base)], -1)
        c = do.norm_plain(every[:, self.a.c_off:self.a.c_off + R], self.norm, 1e-5)
        kr = do.rotate_half(every[:, self.a.c_off + R:self.a.g_off], at, self.base)
        k = np.concatenate([(c @ self.uk.T).reshape(n, H, d), np.broadcast_to(kr[:, None], (n, H, r))], -1)
        v = (c @ self.uv.T).reshape(n, H, e)
        o = do.causal_attention(q[n - len(x):], k, v, self.scale, n - len(x))
        return (o * do.sigmoid(x[:, self.a.g_off:])[:, :, None]).reshape(len(x), H * e)


SIZES = [  # heads, dim, rot, vdim, rank: matrix-core sizes ...
    (4, 32, 16, 32, 64), (8, 96, 32, 64, 96), (3, 20, 6, 12, 24), (16, 32, 64, 32, 512), (20, 64, 64, 48, 200), (33, 32, 8, 160, 256),
    (1, 96, 2, 7, 128), (1, 1, 2, 1, 1), (2, 300, 10, 20, 60),
    # ... and others
    (2, 32, 128, 32, 64), (2, 64, 32, 32, 640)]


@pytest.mark.parametrize("size", SIZES)
@pytest.mark.parametrize("fp32", [False, True])
def test_latent_attention_in_any_portions_and_decoded(t12, oracle, size, fp32):
    A = Latent(t12, oracle, *size, fp32=fp32)
    assert bool(A.a.matrix) == (not fp32 and size[2] <= 64 and size[4] <= 512)
    n = 150
    x = A.inputs(n, sum(size))
    want = A.oracle(x)
    tol = 2e-5 if fp32 else 2e-2
    for cuts in ([150], [64, 64, 22], [2, 31, 33, 1, 50, 33], [2] * 75):
        at = 0
        for c in cuts:
            got = A.feed(x[at:at + c], range(at, at + c), 0)
            assert off(got, want[at:at + c], want) < tol, (cuts[:6], at)
            at += c
    A.feed(x[:61], range(61), 0)
    for i in range(61, n):
        assert off(A.feed(x[i:i + 1], [i], [0]), want[i:i + 1], want) < tol, i


@pytest.mark.parametrize("fp32", [False, True])
def test_one_key_that_stands_out(t12, oracle, fp32):
    """Queries that point at one key: near, far, at the borders of the cache's blocks, the first ones -- and at the next token, which
    must not be seen."""
    R, n = 64, 200
    eye = np.eye(R)
    A = Latent(t12, oracle, 2, R, 16, R, R, fp32=fp32, scale=1.0, uk=np.tile(eye, (2, 1)), uv=np.tile(eye, (2, 1)))
    x = A.inputs(n, 1)
    c = do.norm_plain(x[:, A.a.c_off:A.a.c_off + R], A.norm, 1e-5)
    rng = np.random.default_rng(2)
    target = []
    for i in range(n):
        cand = sorted({0, 1, 31, 32, 63, 64, 65, i, i - 1, i + 1, i - 31, i - 32, i - 33, i // 32 * 32, i // 32 * 32 - 1} & set(range(min(i + 2, n))))
        target.append(cand[int(rng.integers(len(cand)))])
    q = np.zeros((n, 2, R + 16))
    q[:, :, :R] = 0.6 * c[target][:, None]
    x[:, :2 * (R + 16)] = bf16(q.reshape(n, -1))
    x[:, A.a.g_off:] = 30.0
    want = A.oracle(x)
    seen = np.array(target) <= np.arange(n)
    near = lambda w: np.abs(w[:, :R] - c[target] @ A.uv[:R].T).max(1)
    assert near(want)[seen].max() < 1e-3 * np.abs(want).max() and near(want)[~seen].min() > 0.1
    tol = 2e-5 if fp32 else 2e-2
    got = np.concatenate([A.feed(x[a:b], range(a, b), 0) for a, b in ((0, 97), (97, 99), (99, 200))])
    assert rel_err(got, want) < tol
    A.feed(x[:40], range(40), 0)
    got = np.concatenate([A.feed(x[i:i + 1], [i], [0]) for i in range(40, n)])
    assert rel_err(got, want[40:]) < tol


@pytest.mark.parametrize("size", [(4, 32, 16, 32, 64), (16, 64, 64, 64, 512), (40, 32, 32, 32, 128)])
def test_long_contexts_are_split_over_workgroups(t12, oracle, size):
    """Decode steps and short portions behind 2000 tokens: stretches of keys in several workgroups, put together."""
    A = Latent(t12, oracle, *size, rows=700, scale=0.6)
    x = A.inputs(2110, 5)
    for s in range(0, 2100, 700):
        A.feed(x[s:s + 700], range(s, s + 700), 0)
    at = 2100
    for step in (1, 2, 1, 5, 1):
        want = A.oracle(x[at:at + step], x[:at], at)
        rows = [0] if step == 1 else 0
        a, b = (A.feed(x[at:at + step], range(at, at + step), rows) for _ in range(2))
        assert rel_err(a, want) < 4e-2 and np.array_equal(a, b)
        at += step


def test_rotation_far_into_a_sequence(t12, oracle):
    """Angles of large positions, in 32 bits: the cache before the first row holds zeros, which are keys of score 0."""
    A = Latent(t12, oracle, 2, 16, 32, 16, 32, fp32=True, positions=30100)
    x = A.inputs(6, 8)
    first = 30000
    got = A.feed(x, range(first, first + 6), 0)
    past = np.zeros((first, A.ld))
    assert rel_err(got, A.oracle(x, past, first)) < 2e-2               # (fp32 angles: 30000 x 2^-24)


def test_latent_rows_of_their_own(t12, oracle):
    B = 5
    A = Latent(t12, oracle, 6, 32, 16, 24, 96, regions=B)
    lens = [50, 0, 33, 31, 64]
    seqs = [A.inputs(m + 4, 60 + m) for m in lens]
    A.feed(A.inputs(90, 1), range(90), 1)                              # somebody was in region 1 before
    for b in range(B):
        if lens[b]:
            A.feed(seqs[b][:lens[b]], range(lens[b]), b)
    want = [A.oracle(s) for s in seqs]
    for s in range(4):
        got = A.feed(np.stack([seqs[b][lens[b] + s] for b in range(B)]), [m + s for m in lens], list(range(B)))
        for b in range(B):
            assert off(got[b], want[b][lens[b] + s], want[b]) < 2e-2, (b, s)


# ------------------------------------------------------------------------------------------------- layer pieces
def test_normed_embedding(t12):
    rng = np.random.default_rng(0)
    (b, v), w = bits_and_values(rng.standard_normal((11, 50))), 1 + rng.standard_normal(50)
    tok = [3, 0, 10, 11, -1, 3]
    table, td, wd, out = up(b.view(np.int16), torch.int16), up(np.array(tok), torch.int32), up(w), torch.empty((6, 50), device=dev())
    t12.check(t12.lib.t12_embed_norm(table.data_ptr(), 11, td.data_ptr(), wd.data_ptr(), 1e-5, out.data_ptr(), 50, 6, t12.current_stream()))
    want = np.stack([do.rms(v[t], 1e-5) * w if 0 <= t < 11 else np.zeros(50) for t in tok])
    assert rel_err(host(out), want) < 1e-6


@pytest.mark.parametrize("width, n, splits", [(64, 5, 1), (50, 3, 4), (2048, 9, 1), (4096, 2, 8), (8192, 2, 3), (6000, 2, 1), (9000, 2, 2), (1, 4, 1)])
@pytest.mark.parametrize("fp32", [False, True])
def test_norms_around_a_sublayer(t12, width, n, splits, fp32):
    rng = np.random.default_rng(width)
    y, res = rng.standard_normal((splits, n, width)), 3 * rng.standard_normal((n, width))
    pw, nw = 1 + 0.3 * rng.standard_normal((2, width))
    yd, rd, pd, nd = up(y), up(res), up(pw), up(nw)
    x = torch.empty((n, width), device=dev())
    h = torch.empty((n, width), dtype=torch.float32 if fp32 else torch.bfloat16, device=dev())
    part = t12.GemmPartials(yd.data_ptr(), splits, width, n * width)
    t12.check(t12.lib.t12_post_norm_add(yd.data_ptr(), C.byref(part) if splits > 1 else None, rd.data_ptr(), pd.data_ptr(), nd.data_ptr(),
                                        1e-5, x.data_ptr(), h.data_ptr(), int(fp32), width, n, t12.current_stream()))
    want = res + do.rms(y.sum(0), 1e-5) * pw
    assert rel_err(host(x), want) < 2e-6
    assert rel_err(host(h), do.rms(want, 1e-5) * nw) < (3e-6 if fp32 else 5e-3)
    if splits == 1:                                                    # in place
        t12.check(t12.lib.t12_post_norm_add(yd.data_ptr(), None, rd.data_ptr(), pd.data_ptr(), nd.data_ptr(), 1e-5, yd.data_ptr(), h.data_ptr(),
                                            int(fp32), width, n, t12.current_stream()))
        assert torch.equal(yd[0], x)


def test_gated_units(t12):
    rng = np.random.default_rng(1)
    g, u = 4 * rng.standard_normal((2, 1003))
    gd, ud = up(g), up(u)
    for glu, want in ((t12.Glu(1.5, 1.702, 1.0), do.clamped_glu(g, u, 1.5)), (t12.Glu(float("inf"), 1.0, 0.0), g * do.sigmoid(g) * u),
                      (t12.Glu(0.0, 1.702, 1.0), do.clamped_glu(g, u, 0.0))):
        for fp32 in (True, False):
            out = torch.empty(1003, dtype=torch.float32 if fp32 else torch.bfloat16, device=dev())
            t12.check(t12.lib.t12_glu(gd.data_ptr(), ud.data_ptr(), C.byref(glu), out.data_ptr(), int(fp32), 1003, t12.current_stream()))
            assert rel_err(host(out), want) < (1e-6 if fp32 else 5e-3)


@pytest.mark.parametrize("M, K", [(96, 64), (130, 1024), (64, 2064), (1000, 4096)])
def test_gated_decode_gemv(t12, oracle, M, K):
    rng = np.random.default_rng(M + K)
    (ta, wa), (tb, wb) = (packed(t12, oracle, rng.standard_normal((M, K)) * 1.5 / np.sqrt(K)) for _ in range(2))
    xb, xv = bits_and_values(rng.standard_normal(K))
    xd, out = up(xb.view(np.int16), torch.int16), torch.empty(M, dtype=torch.bfloat16, device=dev())
    g, u, glu = ta.segment(None), tb.segment(None), t12.Glu(0.8, 1.702, 1.0)
    t12.check(t12.lib.t12_gemv_glu(C.byref(g), C.byref(u), C.byref(glu), xd.data_ptr(), K, out.data_ptr(), t12.current_stream()))
    assert rel_err(host(out), do.clamped_glu(wa @ xv, wb @ xv, 0.8)) < 5e-3


@pytest.mark.parametrize("M, K", [(96, 64), (130, 1024), (64, 2064), (1000, 4096), (40, 8192)])
def test_decode_gemv_with_the_norms_around_a_sublayer(t12, oracle, M, K):
    rng = np.random.default_rng(M * K)
    (ta, wa), (tb, wb) = (packed(t12, oracle, rng.standard_normal((M, K)) / np.sqrt(K)) for _ in range(2))
    y, res = rng.standard_normal(K), 2 * rng.standard_normal(K)
    yd, rd, out, hid = up(y), up(res), torch.empty(M, device=dev()), torch.empty(K, device=dev())
    lib, st = t12.lib, t12.current_stream()
    s = res + do.norm_one_gain(y, 0.7, 1e-5)
    h = do.norm_one_gain(s, 1.3, 1e-5)
    seg = (t12.Segment * 1)(ta.segment(out))
    t12.check(lib.t12_gemv_gain_norm(seg, 1, yd.data_ptr(), rd.data_ptr(), 0.7, 1.3, 1e-5, hid.data_ptr(), K, st))
    assert rel_err(host(hid), s) < 2e-6 and rel_err(host(out), wa @ h) < 1e-2
    o16, hid2 = torch.empty(M, dtype=torch.bfloat16, device=dev()), torch.empty(K, device=dev())
    g, u, glu = ta.segment(None), tb.segment(None), t12.Glu(0.8, 1.702, 1.0)
    t12.check(lib.t12_gemv_glu_gain_norm(C.byref(g), C.byref(u), C.byref(glu), yd.data_ptr(), rd.data_ptr(), 0.7, 1.3, 1e-5, hid2.data_ptr(), K,
                                         o16.data_ptr(), st))
    assert torch.equal(hid, hid2) and rel_err(host(o16), do.clamped_glu(wa @ h, wb @ h, 0.8)) < 2e-2


@pytest.mark.parametrize("M, K, B", [(200, 128, 6), (12400, 128, 70), (12400, 64, 300), (300, 256, 100)])
def test_gated_product_over_a_batch(t12, oracle, M, K, B):
    rng = np.random.default_rng(M + B)
    (ta, wa), (tb, wb) = (packed(t12, oracle, rng.standard_normal((M, K)) * 1.5 / np.sqrt(K)) for _ in range(2))
    xb, xv = bits_and_values(rng.standard_normal((B, K)))
    xd = up(xb.view(np.int16), torch.int16)
    out = torch.zeros((B, M), dtype=torch.bfloat16, device=dev())
    g, u, glu = ta.segment(None), tb.segment(None), t12.Glu(1.1, 1.702, 1.0)
    rc = t12.lib.t12_gemm_glu(C.byref(g), C.byref(u), C.byref(glu), xd.data_ptr(), K, K, B, out.data_ptr(), M, t12.current_stream())
    assert rc == (1 if M == 300 else 0)
    if rc == 0:
        assert rel_err(host(out), do.clamped_glu(xv @ wa.T, xv @ wb.T, 1.1)) < 5e-3


def test_host_side_refusals(t12):
    lib, m, a = t12.lib, t12.MatrixMemory(), t12.LatentAttn()
    m.heads, m.dim, m.vdim = 1, 513, 8
    assert lib.t12_memory_plan(C.byref(m), 8) == -1
    m.dim = 512
    assert lib.t12_memory_plan(C.byref(m), 8) == 0 and m.dim_p == 512
    assert lib.t12_matrix_memory(C.byref(m), None, None, 0, None, 1, 0, 0, None, None, 0, 0, None) == -1
    a.heads, a.dim, a.rot_dim, a.vdim, a.rank, a.elem_bytes = 2, 16, 5, 16, 32, 2
    assert lib.t12_latent_plan(C.byref(a), 100, 8) == -1               # an odd rotated part
    a.rot_dim = 6
    assert lib.t12_latent_plan(C.byref(a), 100, 8) == 0 and a.rank_p == 64 and a.row_p == 128
    assert lib.t12_latent_attention(C.byref(a), None, 0, None, 1, 0, 0, None, None, 0, 0, None) == -1
    assert lib.t12_post_norm_add(None, None, None, None, None, 0.0, None, None, 0, 8, 1, None) == -1
