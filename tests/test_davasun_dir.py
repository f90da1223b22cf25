"""CPU: what load_model's host-only check says about Davasun directories -- checkpoints that are right, and ones with a missing
or misshapen tensor, a broken container or an impossible configuration."""
import copy
import json

import pytest

from davasun_util import config, latent, mlstm, tensors, write_checkpoint
from test_gamilorn_dir import check

CFG = config([mlstm(), latent(), latent(heads=2, rank=40, ff=0), mlstm(ff=32)], width=48, loop=(0, 2, 3))


@pytest.fixture
def ckpt(t12, tmp_path):
    write_checkpoint(tmp_path, CFG, tensors(CFG, 1))
    return tmp_path


def test_a_whole_checkpoint_is_consistent(t12, ckpt):
    assert check(t12, ckpt) == (True, "")


@pytest.mark.parametrize("name", ["embed", "embed.norm", "head", "final.norm", "l0.norm1b", "l1.norm2", "l0.mix.i.b", "l3.mix.norm",
                                  "l1.mix.dkv", "l1.mix.dkv.norm", "l2.mix.uk", "l1.mix.uv", "l2.mix.g", "l3.mlp.gate"])
def test_missing_and_misshapen_tensors_are_named(t12, tmp_path, name):
    t = tensors(CFG, 1)
    x = t.pop(name)
    write_checkpoint(tmp_path / "a", CFG, t)
    ok, msg = check(t12, tmp_path / "a")
    assert not ok and name in msg
    t[name] = x[:-1] if x.ndim else x.reshape(1)               # a gain is a number, not a list of one
    write_checkpoint(tmp_path / "b", CFG, t)
    ok, msg = check(t12, tmp_path / "b")
    assert not ok and name in msg


def test_a_layer_without_feed_forward_needs_none_of_its_tensors(t12, tmp_path):
    t = tensors(CFG, 1)
    assert not any(k.startswith(("l0.mlp", "l2.mlp")) or k in ("l0.norm2", "l2.norm2b") for k in t)
    write_checkpoint(tmp_path, CFG, t)
    assert check(t12, tmp_path)[0]


@pytest.mark.parametrize("edit, word", [
    (lambda c: c["layers"][0].update(type="parallel"), "parallel"),
    (lambda c: c["layers"][1]["mlp"].update(kind="experts"), "experts"),
    (lambda c: c["layers"][1]["mlp"].pop("limit"), "limit"),
    (lambda c: c["layers"][0]["mixer"].pop("gate_cap"), "gate_cap"),
    (lambda c: c["layers"][0]["mixer"].update(gate_cap=0), "gate_cap"),
    (lambda c: c["layers"][0]["mixer"].update(dim=513), "dim"),
    (lambda c: c["layers"][1]["mixer"].update(rot_dim=15), "odd"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=8), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"].pop("rot"), "rot"),
    (lambda c: c["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][1]["mixer"].update(kv_rank=0), "kv_rank"),
    (lambda c: c["loop"].update(stop=5), "stop"),
    (lambda c: c["loop"].update(times=0), "times"),
    (lambda c: c.update(loop={"start": 2, "stop": 1, "times": 1}), "stop"),
    (lambda c: c.update(layers=[]), "layers"),
    (lambda c: c.pop("logit_scale"), "logit_scale"),
    (lambda c: c["norm"].pop("eps"), "eps"),
])
def test_impossible_configurations(t12, ckpt, edit, word):
    c = copy.deepcopy(CFG)
    edit(c)
    (ckpt / "config.json").write_text(json.dumps(c))
    ok, msg = check(t12, ckpt)
    assert not ok and word in msg


def test_a_model_without_a_loop(t12, tmp_path):
    for drop in (True, False):
        c = copy.deepcopy(CFG)
        c["loop"] = None
        if drop:
            c.pop("loop")
        write_checkpoint(tmp_path / str(drop), c, tensors(c, 1))
        assert check(t12, tmp_path / str(drop)) == (True, "")


def test_directory_without_tensors(t12, tmp_path):
    (tmp_path / "config.json").write_text(json.dumps(CFG))
    ok, msg = check(t12, tmp_path)
    assert not ok and "model.safetensors" in msg
