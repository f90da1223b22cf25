"""GPU: Davasun models through the engine's own entry points -- load, prompts in portions, decoding, batches, sampling,
generation -- against the float64 oracle on the same weights."""
import importlib
import json
import os
import struct
import subprocess
import sys

import numpy as np
import pytest
import torch  # noqa: F401  (before the library: its HIP runtime is then the process's only one)

from davasun_util import config, error, latent, mlstm, tensors, write_checkpoint
from oracle import davasun_oracle as do

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

# "mixed": both mixers with unlike sizes, with and without feed-forwards, a loop over layers of both kinds in the middle;
# "odd": nothing is a multiple of anything, the loop over everything; "plain": no loop, attention first, one
# head, wide latents; "memory": no attention at all.
MODELS = {
    "mixed": (config([mlstm(), mlstm(heads=3, dim=40, vdim=16, cap=15.0, ff=72, limit=3.0), latent(heads=6, dim=32, rot=24, vdim=40, rank=96),
                      latent(heads=2, dim=64, rot=32, vdim=64, rank=128, base=10000.0, ff=0), mlstm(heads=1, dim=64, vdim=96, cap=4.0)],
                     width=128, vocab=203, loop=(1, 3, 2), logit_scale=2.5), 11),
    "odd": (config([latent(heads=3, dim=20, rot=6, vdim=12, rank=28, ff=52, limit=0.7), mlstm(heads=5, dim=9, vdim=21, ff=0), mlstm(heads=1, dim=14, vdim=33)],
                   width=72, vocab=61, loop=(0, 3, 3), logit_scale=1.0), 12),
    "plain": (config([latent(heads=1, dim=128, rot=64, vdim=160, rank=300, ff=256), mlstm(heads=2, dim=160, vdim=144, ff=64), mlstm(heads=4, dim=32, vdim=32)],
                     width=256, vocab=300, eps=1e-3, logit_scale=4.0), 13),
    "memory": (config([mlstm(heads=2, dim=48, vdim=48)], width=96, vocab=120, loop=(0, 1, 4)), 14),
}


@pytest.fixture(scope="module", params=list(MODELS))
def model(request, t12, tmp_path_factory):
    cfg, seed = MODELS[request.param]
    path = str(tmp_path_factory.mktemp("davasun"))
    t = write_checkpoint(path, cfg, tensors(cfg, seed))
    return path, cfg, t


@pytest.fixture(autouse=True)
def plain_environment(monkeypatch):
    for name in ("TURBO_CTX", "TURBO_NO_FUSE", "TURBO_NO_PIPELINE"):       # other tests of the process may have set them
        monkeypatch.delenv(name, raising=False)


TOL = {False: 4e-2, True: 5e-5}


def off(cfg, t, tok, got, want, fp32=False):
    """Largest error of a row over what that row may have: the tolerance, or in bf16 three times what rounding-sized noise on the
    matrices does to the oracle there (a normaliser that nearly cancels, and a head's output over its own RMS, amplify).
    tok: the sequence up to the rows' end; got, want: its last rows."""
    err = np.sqrt(np.mean((got - want) ** 2, axis=-1)) / np.sqrt(np.mean(np.asarray(want) ** 2))
    if fp32 or (err < TOL[False]).all():
        return float((err / TOL[fp32]).max())
    clean = do.forward(cfg, t, tok)
    may = np.full(len(tok), TOL[False])
    for seed in range(6):
        rng = np.random.default_rng(seed)
        noisy = dict(t)
        for name in noisy:
            if noisy[name].ndim == 2:
                noisy[name] = t[name] * (1 + 2 ** -9 * rng.standard_normal(t[name].shape))
        d = do.forward(cfg, noisy, tok) - clean
        may = np.maximum(may, 3 * np.sqrt(np.mean(d ** 2, axis=-1)) / np.sqrt(np.mean(np.asarray(want) ** 2)))
    return float((err / may[len(tok) - len(err):]).max())


def ids(cfg, n, seed):
    return [int(x) for x in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


@pytest.mark.parametrize("fp32", [True, False])
def test_whole_prompts_and_portions(t12, model, fp32):
    path, cfg, t = model
    tok = ids(cfg, 170, 1)
    want = do.forward(cfg, t, tok)
    for rows in (0, 16):                                     # 16: small passes, the tightest rings
        eng = t12.Engine.load(path, prompt_rows=rows, fp32=fp32)
        try:
            assert eng.family == "davasun" and eng.n_vocab == cfg["vocab"]
            for cuts in ([170], [2, 31, 1, 64, 33, 39], [2] * 85, [1] * 40 + [130], [100] + [1] * 70):
                eng.set_positions([0])                        # the same region again, whatever it held
                at, parts = 0, []
                for c in cuts:
                    parts.append(eng.prefill_logits(0, tok[at:at + c]))
                    at += c
                assert off(cfg, t, tok, np.concatenate(parts), want, fp32) < 1, (rows, cuts[:6])
        finally:
            eng.close()


def stepped(t12, path, cfg, tok):
    """Logits of every step of a batch-1 state, one token at a time."""
    eng = t12.Engine.load(path)
    try:
        got = []
        for x in tok:
            eng.forward([x])
            got.append(eng.logits(cfg["vocab"]).cpu().numpy()[0])
        return np.stack(got)
    finally:
        eng.close()


@pytest.mark.parametrize("fused", [True, False])
def test_steps_of_one_sequence(t12, model, fused, monkeypatch):
    path, cfg, t = model
    tok = ids(cfg, 60, 2)
    if not fused:
        monkeypatch.setenv("TURBO_NO_FUSE", "1")
    assert off(cfg, t, tok, stepped(t12, path, cfg, tok), do.forward(cfg, t, tok)) < 1


def test_decode_with_a_large_vocabulary(t12, tmp_path):
    """Its head reads an input normed by a kernel of its own; smaller ones norm it in the product's prologue."""
    for tail in (mlstm(), latent(ff=0)):
        cfg = config([latent(), tail], width=80, vocab=8200)
        path = str(tmp_path / tail["type"])
        t = write_checkpoint(path, cfg, tensors(cfg, 17))
        tok = ids(cfg, 40, 7)
        assert off(cfg, t, tok, stepped(t12, path, cfg, tok), do.forward(cfg, t, tok)) < 1


def test_picked_places_equal_all_places(t12, model):
    path, cfg, _ = model
    tok = ids(cfg, 90, 3)
    eng = t12.Engine.load(path, prompt_rows=32)
    try:
        every = eng.prefill_logits(0, tok)
        eng.set_positions([0])
        pick = [0, 31, 32, 50, 89]
        assert error(eng.prefill_logits(0, tok, pick), every[pick]) < 1e-2
        eng.set_positions([0])
        assert eng.prefill_logits(0, tok, []).shape == (0, cfg["vocab"])
        eng.set_positions([0])
        eng.prefill(0, tok)                                   # the last place's logits stay in the state
        assert error(eng.logits(cfg["vocab"]).cpu().numpy(), every[-1:]) < 1e-2
        with pytest.raises(t12.T12Error):
            eng.prefill_logits(0, tok[:4], [2, 1])
    finally:
        eng.close()


@pytest.mark.parametrize("fp32", [True, False])
def test_long_decoding(t12, model, fp32):
    path, cfg, t = model
    tok = ids(cfg, 290, 4)
    want = do.forward(cfg, t, tok)
    eng = t12.Engine.load(path, prompt_rows=8, fp32=fp32)
    try:
        eng.prefill_logits(0, tok[:20])
        got = np.concatenate([eng.prefill_logits(0, [x]) for x in tok[20:]])
        assert off(cfg, t, tok, got, want[20:], fp32) < 1
    finally:
        eng.close()


def test_unequal_sequences_in_a_batch_against_each_alone(t12, model):
    path, cfg, t = model
    lens, steps = [33, 1, 70, 12, 5], 12
    seqs = [ids(cfg, n + steps, 20 + i) for i, n in enumerate(lens)]
    want = [do.forward(cfg, t, s) for s in seqs]
    eng = t12.Engine.load(path, batch=len(lens), per_sequence=120, prompt_rows=24)
    try:
        for again in range(2):                                # the second time every region is one that was used before
            order = [2, 0, 4, 1, 3] if again else range(5)
            eng.set_positions([0] * 5)
            for b in order:
                got = eng.prefill_logits(b, seqs[b][:lens[b]])
                assert off(cfg, t, seqs[b][:lens[b]], got, want[b][:lens[b]]) < 1, b
            assert eng.positions() == lens
            for s in range(steps):
                eng.forward([seqs[b][lens[b] + s] for b in range(5)])
                got = eng.logits(cfg["vocab"]).cpu().numpy()
                for b in range(5):
                    assert off(cfg, t, seqs[b][:lens[b] + s + 1], got[b:b + 1], want[b][lens[b] + s:lens[b] + s + 1]) < 2, (b, s)
            seqs, lens, want = [seqs[i] for i in (1, 2, 3, 4, 0)], [lens[i] for i in (1, 2, 3, 4, 0)], [want[i] for i in (1, 2, 3, 4, 0)]
    finally:
        eng.close()


def test_one_sequence_of_a_batch_restarts_while_the_others_go_on(t12, model):
    path, cfg, t = model
    a, b, c = ids(cfg, 50, 30), ids(cfg, 40, 31), ids(cfg, 30, 32)
    eng = t12.Engine.load(path, batch=2, per_sequence=100)
    try:
        eng.prefill(0, a[:40])
        eng.prefill(1, b[:39])
        eng.forward([a[40], b[39]])
        eng.set_positions([41, 0])                            # sequence 1 is done; its slot takes a new one
        eng.prefill(1, c[:20])
        wa, wc = do.forward(cfg, t, a), do.forward(cfg, t, c)
        for s in range(9):
            eng.forward([a[41 + s], c[20 + s]])
            got = eng.logits(cfg["vocab"]).cpu().numpy()
            assert off(cfg, t, a[:42 + s], got[:1], wa[41 + s:42 + s]) < 2 and off(cfg, t, c[:21 + s], got[1:], wc[20 + s:21 + s]) < 2
    finally:
        eng.close()


def test_lock_step_copies_on_one_region(t12, model):
    path, cfg, t = model
    tok = ids(cfg, 40, 5)
    want = do.forward(cfg, t, tok)
    eng = t12.Engine.load(path, batch=3)
    try:
        eng.prefill(0, tok[:30])
        assert eng.positions() == [30] * 3
        assert off(cfg, t, tok[:30], eng.logits(cfg["vocab"]).cpu().numpy()[1:2], want[29:30]) < 1
        for s in range(30, 40):
            eng.forward([tok[s]] * 3)
            got = eng.logits(cfg["vocab"]).cpu().numpy()
            assert np.array_equal(got[0], got[2]) and off(cfg, t, tok[:s + 1], got[:1], want[s:s + 1]) < 1
    finally:
        eng.close()


def oracle_greedy(cfg, t, prompt, n):
    st, out = do.State(cfg), []
    last = do.forward(cfg, t, prompt, st)[-1]
    gaps = []
    for _ in range(n):
        top = np.sort(last)[-2:]
        gaps.append(top[1] - top[0])
        out.append(int(last.argmax()))
        last = do.forward(cfg, t, out[-1:], st)[-1]
    return out, gaps


def test_greedy_generation(t12, model):
    """generate() of a 32-bit state gives the oracle's stream (up to a tie of its two best ids)."""
    path, cfg, t = model
    prompt = ids(cfg, 15, 6)
    want, gaps = oracle_greedy(cfg, t, prompt, 40)
    sure = next((i for i, g in enumerate(gaps) if g < 1e-3), 40)
    stop = want.index(2) if 2 in want else 40
    eng = t12.Engine.load(path, fp32=True)
    try:
        got = eng.generate(prompt, 40)
        n = min(sure, stop)
        assert n >= 10 and got[:n] == want[:n]
        if sure > stop:
            assert len(got) == stop
    finally:
        eng.close()


def test_a_stop_id_takes_the_step_ahead_back(t12, model):
    """The pipelined loop has already run the stop id through the layers when it stops: state, positions and logits must be
    those from before it, and decoding goes on from there."""
    path, cfg, t = model
    prompt = ids(cfg, 25, 7)
    for fp32 in (False, True):
        eng = t12.Engine.load(path, fp32=fp32)
        try:
            eng.prefill(0, prompt)
            free = eng.decode(16)
            cut = next(i for i in range(4, 16) if free[i] not in free[:i])
            eng.set_positions([0])
            eng.prefill(0, prompt)
            assert eng.decode_until(16, free[cut]) == free[:cut]
            assert eng.positions() == [25 + cut]
            want = do.forward(cfg, t, prompt + free[:cut])[-1:]
            assert off(cfg, t, prompt + free[:cut], eng.logits(cfg["vocab"]).cpu().numpy(), want, fp32) < 2
            assert eng.sample() == [free[cut]]
            tail = ids(cfg, 6, 8)
            got = np.concatenate([eng.prefill_logits(0, [x]) for x in tail])
            assert off(cfg, t, prompt + free[:cut] + tail, got, do.forward(cfg, t, prompt + free[:cut] + tail)[-6:], fp32) < 2
        finally:
            eng.close()


def test_decode_all_matches_step_by_step(t12, model):
    path, cfg, _ = model
    eng = t12.Engine.load(path, batch=3, per_sequence=80)
    try:
        prompts = [ids(cfg, n, 40 + n) for n in (9, 20, 2)]
        for b in range(3):
            eng.prefill(b, prompts[b])
        fast = eng.decode_all(12)
        eng.set_positions([0] * 3)
        for b in range(3):
            eng.prefill(b, prompts[b])
        slow = []
        for _ in range(12):
            slow.append(eng.sample())
            eng.forward(slow[-1])
        assert fast == slow
    finally:
        eng.close()


def test_saved_directory_loads_to_the_same_model(t12, model, tmp_path):
    path, cfg, _ = model
    tok = ids(cfg, 30, 9)
    a = t12.Engine.load(path)
    try:
        a.save(str(tmp_path))
        want = a.prefill_logits(0, tok)
    finally:
        a.close()
    assert not os.path.exists(tmp_path / "model.safetensors")
    b = t12.Engine.load(str(tmp_path))
    try:
        assert np.array_equal(b.prefill_logits(0, tok), want)
    finally:
        b.close()
    os.remove(tmp_path / "l0.mix.in.sm.bin")
    with pytest.raises(t12.T12Error):
        t12.Engine.load(str(tmp_path))


def test_convert_packs_a_checkpoint(t12, model, tmp_path):
    path, cfg, _ = model
    conv = importlib.import_module("turbo_lossless_amd.convert")
    stats = conv.convert(path, str(tmp_path / "out"))
    assert stats["l0.mix.in"][1] == cfg["width"] and stats["head"][:2] == (cfg["vocab"], cfg["width"])
    eng = t12.Engine.load(str(tmp_path / "out"))
    eng.close()


def test_what_a_recurrent_model_cannot_do(t12, model, monkeypatch):
    path, cfg, _ = model
    monkeypatch.setenv("TURBO_CTX", "300")
    eng = t12.Engine.load(path)
    try:
        eng.prefill(0, ids(cfg, 10, 1))
        with pytest.raises(t12.T12Error, match="shifted"):
            eng.shift_context(10, 5)
        eng.set_positions([4])
        with pytest.raises(t12.T12Error, match="recurrent"):
            eng.forward([1])
        eng.set_positions([0])
        eng.forward([1])
        with pytest.raises(t12.T12Error, match="exceeds"):
            eng.prefill(0, [1] * 300)
    finally:
        eng.close()


def test_chat_turns_until_the_context_is_full(t12, model, monkeypatch):
    """Turns continue one sequence as generate() of everything at once would; nothing is ever discarded."""
    path, cfg, t = model
    context = 200
    monkeypatch.setenv("TURBO_CTX", str(context))
    eng = t12.Engine.load(path, fp32=True)
    try:
        pos, fed = 0, []
        for turn in range(3):
            new = ids(cfg, 9, 20 + turn)
            out, pos, dropped = eng.chat_turn(pos, new, 7, -1, 2, prompt_rows=4)
            fed += new + out + [2]
            assert dropped == 0 and pos == len(fed)
        got = eng.prefill_logits(0, new, [8])
        assert error(got, do.forward(cfg, t, fed + new)[-1:]) < TOL[True]
        pos += 9
        out, end, _ = eng.chat_turn(pos, [1] * (context - pos - 4), 50, -1, 2, prompt_rows=64)
        assert len(out) <= 3 and end <= context       # cut to the room that was left
        pos = end
        with pytest.raises(t12.T12Error, match="do not fit"):
            eng.chat_turn(pos, [1] * (context - pos + 1), 4, -1, 2, prompt_rows=64)
    finally:
        eng.close()


def test_a_shorter_context_can_be_asked_for(t12, model, monkeypatch):
    path, cfg, _ = model
    monkeypatch.setenv("TURBO_CTX", "40")
    eng = t12.Engine.load(path)
    try:
        eng.prefill(0, ids(cfg, 40, 1))
        with pytest.raises(t12.T12Error, match="exceeds"):
            eng.forward([0])
    finally:
        eng.close()


def test_trace_replay_program(t12, model, tmp_path):
    path, cfg, t = model
    a, b = ids(cfg, 30, 50), ids(cfg, 20, 51)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:17], "want": [16, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b, "want": []}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "c", "tokens": b[:5], "want": [4]}, {"id": "a", "tokens": a[17:18], "want": [0]}], "end": ["c"]},
             {"step": 3, "entries": [{"id": "a", "tokens": a[18:], "want": list(range(12))}], "end": ["a"]}]
    wa, wb = do.forward(cfg, t, a), do.forward(cfg, t, b[:5])
    want = {0: wa[[16, 3]], 2: np.stack([wb[4], wa[17]]), 3: wa[18:]}
    for dtype in ("bfloat16", "float32"):
        out = tmp_path / dtype
        out.mkdir()
        r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out", str(out),
                            "--max-tokens", "64"], input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True,
                           timeout=100)
        assert r.returncode == 0, r.stderr[-2000:]
        done = [ln for ln in r.stdout.splitlines() if ln.startswith("done ")]
        assert done == ["done %d" % i for i in range(4)]
        assert not (out / "1.f32").exists()
        for s, w in want.items():
            got = np.fromfile(out / ("%d.f32" % s), "<f4").reshape(w.shape)
            assert error(got, w) < (5e-5 if dtype == "float32" else 0.25), (dtype, s)


def test_synthetic_models(t12):
    cfg = config([mlstm(heads=4, dim=64, vdim=128, ff=512), latent(heads=8, dim=64, rot=32, vdim=64, rank=128, ff=512)], width=512, vocab=1000, loop=(0, 1, 2))
    eng = t12.Engine.synthetic_davasun(cfg, batch=2, per_sequence=64)
    try:
        a = eng.prefill_logits(0, list(range(20)))
        b = eng.prefill_logits(1, list(range(20)))
        assert np.isfinite(a).all() and np.array_equal(a, b) and a.std() > 0
    finally:
        eng.close()
