"""Siterax without a GPU: the configuration reader, the registry, the rotary table, and the oracle itself (identities, and that a window one key off, a lost sink, a lost
injection or a wrong rotation really shows in its logits: what the GPU tests' tolerances rely on)."""
import copy
import json

import pytest
import torch

from oracle import siterax_oracle as O
from siterax_util import CONFIGS, save_checkpoint, tokens, weights


def test_config_reads_every_size_and_constant():
    from llava_mi355x.siterax import SiteraxConfig
    c = SiteraxConfig.from_dict(CONFIGS["mixed"])
    assert (c.width, c.vocab_size, c.loop, c.residual_mult, c.logit_softcap, c.norm_eps) == (192, 203, (1, 3, 3), 0.7, 20.0, 1e-5)
    a, b, d, e = c.layers
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.ff) == (4, 2, 48, 64, 24, 160) and (a.rot.dims, a.rot.base, a.rot.factor) == (32, 5000.0, 3.0)
    assert (b.window, b.ff, b.rot.factor) == (0, 0, 1.0) and d.rot.dims == 20 and e.window == 7
    assert SiteraxConfig.from_dict(CONFIGS["odd"]).loop == (0, 0, 1)


@pytest.mark.parametrize("where,value", [("type", "recurrence"), ("mlp", {"kind": "experts", "ff": 8})])
def test_config_refuses_what_it_does_not_know(where, value):
    from llava_mi355x.siterax import SiteraxConfig
    c = copy.deepcopy(CONFIGS["mixed"])
    c["layers"][0][where] = value
    with pytest.raises(ValueError):
        SiteraxConfig.from_dict(c)


def test_registry_chooses_the_family(tmp_path):
    from llava_mi355x import registry
    save_checkpoint(str(tmp_path / "s"), CONFIGS["odd"], {"embed": torch.zeros(2, 2)})
    assert registry.family_of(str(tmp_path / "s")).name == "siterax"
    for d in ({"model_type": "llava"}, {"architectures": ["LlavaLlamaForCausalLM"]}):
        (tmp_path / "config.json").write_text(json.dumps(d))
        assert registry.family_of(str(tmp_path)).name == "llava"
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "something else"}))
    with pytest.raises(ValueError, match="no model family"):
        registry.family_of(str(tmp_path))
    assert dict(registry.iter_checkpoint(str(tmp_path / "s")))["embed"].shape == (2, 2)


def test_rotary_table_is_the_oracles_rotation():
    from llava_mi355x.siterax import RotaryConfig, rotary_table
    t = rotary_table(RotaryConfig(20, 7000.0, 1.5), 300).double()
    rot = {"dims": 20, "base": 7000.0, "scaling": {"factor": 1.5}}
    x = torch.randn(300, 1, 24, dtype=torch.float64)
    want = O.rotate(x, torch.arange(300), rot)
    u, v = x[..., :10], x[..., 10:20]
    c, s = t[:, None, :10], t[:, None, 10:]
    got = torch.cat([u * c - v * s, v * c + u * s, x[..., 20:]], -1)
    assert (got - want).abs().max() < 1e-6


def test_softmax_plus_one_is_a_key_of_score_zero():
    s = torch.randn(3, 5, dtype=torch.float64) * 30
    mask = torch.ones(3, 5, dtype=torch.bool); mask[0, 3:] = False
    ext = torch.cat([s.masked_fill(~mask, float("-inf")), torch.zeros(3, 1, dtype=torch.float64)], -1).softmax(-1)[:, :5]
    assert torch.allclose(O.softmax_plus_one(s, mask), ext)
    big = O.softmax_plus_one(torch.full((1, 2), -900.0, dtype=torch.float64), torch.ones(1, 2, dtype=torch.bool))
    assert big.sum() < 1e-300


def test_layer_runs():
    assert O.layer_runs(CONFIGS["mixed"]) == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    assert O.layer_runs(CONFIGS["odd"]) == [(0, False), (1, False)]
    w, t = weights("single"), tokens("single", 20)
    once = dict(CONFIGS["single"], loop=None)
    assert torch.equal(O.logits(CONFIGS["single"], w, t), O.logits(once, w, t))


def test_prefix_causality():
    w, t = weights("mixed"), tokens("mixed", 60)
    assert torch.allclose(O.logits(CONFIGS["mixed"], w, t)[:31], O.logits(CONFIGS["mixed"], w, t[:31]), atol=1e-12)


@pytest.mark.parametrize("name,change", [
    ("mixed", lambda c: c["layers"][0]["mixer"]["mask"].update(size=23)), ("mixed", lambda c: c["layers"][0]["mixer"]["mask"].update(size=25)),
    ("mixed", lambda c: c["layers"][2]["mixer"]["mask"].update(size=131)), ("mixed", lambda c: c["layers"][2]["mixer"]["rot"].update(dims=18)),
    ("mixed", lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=3.1)), ("mixed", lambda c: c["loop"].update(times=2)),
    ("mixed", lambda c: c.update(logit_softcap=None)), ("mixed", lambda c: c.update(residual_mult=0.71)), ("odd", lambda c: c["layers"][0]["mixer"]["mask"].update(size=2)),
    ("odd", lambda c: c["layers"][1]["mixer"]["mask"].update(size=64)), ("odd", lambda c: c["norm"].update(eps=1e-5)), ("wide", lambda c: c["layers"][0]["mixer"]["mask"].update(size=41))])
def test_a_changed_constant_shows_in_the_logits(name, change):
    w, t = weights(name), tokens(name, 200)
    c = copy.deepcopy(CONFIGS[name])
    change(c)
    a, b = O.logits(CONFIGS[name], w, t), O.logits(c, w, t)
    assert ((a - b).pow(2).mean(-1).sqrt() / a.pow(2).mean().sqrt()).max() > 2e-3          # 100 x the fp32 engine's tolerance


def test_command_lines_parse():
    from llava_mi355x import cli
    a = cli.parse(["--model", "d", "--tokens", "1,2", "--tokens", "3", "--temperature", "0.5"])
    assert a.tokens == ["1,2", "3"] and a.temperature == 0.5
    with pytest.raises(SystemExit):
        cli.parse(["--model", "d"])
