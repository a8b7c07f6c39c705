"""Vizosun without a GPU: the configuration reader, the registry, and the oracle itself (each mechanism against another way to compute it, and that a window one key off, a
lost state, a wrong previous token or a lost pass really shows in its logits: what the GPU tests' tolerances rely on)."""
import copy
import json

import pytest
import torch

from oracle import vizosun_oracle as O
from vizosun_util import CONFIGS, RANKS, save_checkpoint, tokens, weights


def test_config_reads_every_size_and_constant():
    from llava_mi355x.vizosun import BigramConfig, DeltaMixer, LatentMixer, VizosunConfig
    shapes = {k: tuple(v.shape) for k, v in weights("mixed").items()}
    c = VizosunConfig.from_dict(CONFIGS["mixed"], shapes)
    assert (c.width, c.vocab_size, c.loop, c.looped, c.norm_eps) == (136, 211, (1, 3, 3), True, 1e-5) and c.bigram == BigramConfig(101, 7, 13)
    a, b, d, e = c.layers
    assert a.mixer == DeltaMixer(4, 2, 24, 40, 3, *RANKS["mixed"]) and (a.ff, a.experts) == (88, 0)
    assert b.mixer == LatentMixer(3, 40, 20, 50, 36, 1.5 * 40 ** -0.5, 24) and (b.ff, b.experts, b.top) == (40, 5, 2)
    assert (d.ff, d.experts, d.top) == (72, 7, 3) and e.mixer.window == 70
    p = VizosunConfig.from_dict(CONFIGS["plain"], {k: tuple(v.shape) for k, v in weights("plain").items()})
    assert p.bigram is None and p.loop == (0, 2, 2) and p.layers[0].mixer.window == 0
    o = VizosunConfig.from_dict(CONFIGS["odd"], {k: tuple(v.shape) for k, v in weights("odd").items()})
    assert o.loop == (0, 0, 1) and not o.looped and o.layers[1].ff == 0


@pytest.mark.parametrize("where,value", [("type", "attention"), ("mlp", {"kind": "sparse", "ff": 8})])
def test_config_refuses_what_it_does_not_know(where, value):
    from llava_mi355x.vizosun import VizosunConfig
    c = copy.deepcopy(CONFIGS["mixed"])
    c["layers"][0][where] = value
    with pytest.raises(ValueError):
        VizosunConfig.from_dict(c, {k: tuple(v.shape) for k, v in weights("mixed").items()})


def test_registry_chooses_the_family_and_reads_shapes(tmp_path):
    from llava_mi355x import registry
    from llava_mi355x.vizosun import VizosunConfig
    w = weights("odd")
    save_checkpoint(str(tmp_path), CONFIGS["odd"], w)
    assert registry.family_of(str(tmp_path)).name == "vizosun"
    assert registry.checkpoint_shapes(str(tmp_path)) == {k: tuple(v.shape) for k, v in w.items()}
    c = VizosunConfig.from_pretrained(str(tmp_path))
    assert (c.layers[0].mixer.decay_rank, c.layers[0].mixer.gate_rank) == RANKS["odd"]
    assert json.load(open(tmp_path / "config.json"))["architecture"] == "Vizosun"


def test_prefixes_with_state_are_reused_whole_or_not_at_all():
    import numpy as np
    from llava_mi355x.reuse import PrefixCache

    class Holder:
        def close(self):
            pass
    pc = PrefixCache(4, 2)
    h = Holder()
    pc.put(np.arange(6), h)
    assert pc.take(np.array([0, 1, 2, 3, 4, 9, 9]), whole=True) == (None, 0)         # the stored sequence has gone another way
    assert pc.take(np.arange(6), whole=True) == (None, 0)                              # nothing would be left to run
    assert pc.take(np.arange(8), whole=True) == (h, 6)


def test_bigram_rows():
    bg = {"buckets": 10, "mul_prev": 3, "mul_cur": 7}
    assert O.bigram_rows([4, 0, 9], bg) == [10, (4 * 3) % 10, (9 * 7) % 10]


def test_delta_rule_is_a_sum_of_decayed_writes():
    """o_t = sum_s (k_s carried to t) . q_t u_s with u from a triangular solve: another way to the same read-out"""
    g0 = torch.Generator().manual_seed(3)
    T, dk, dv = 12, 5, 3
    r = lambda *s: torch.randn(*s, generator=g0, dtype=torch.float64)
    q, k, v, g, beta = r(T, 1, dk), O.unit(r(T, 1, dk)), r(T, 1, dv), torch.sigmoid(r(T, 1, dk)), torch.sigmoid(r(T, 1))
    got = O.delta_rule(q, k, v, g, beta)[:, 0]
    carry = lambda s, t: torch.stack([g[j, 0] for j in range(s + 1, t + 1)]).prod(0) if t > s else torch.ones(dk, dtype=torch.float64)
    A = torch.eye(T, dtype=torch.float64)
    for t in range(T):
        for s in range(t):
            A[t, s] = beta[t, 0] * (k[t, 0] * carry(s, t) * k[s, 0]).sum()
    u = torch.linalg.solve(A, beta * v[:, 0])
    want = torch.stack([sum((q[t, 0] * carry(s, t) * k[s, 0]).sum() * u[s] for s in range(t + 1)) for t in range(T)])
    assert (got - want).abs().max() < 1e-12


def test_short_conv_is_conv1d():
    x, w = torch.randn(9, 4, dtype=torch.float64), torch.randn(4, 3, dtype=torch.float64)
    want = torch.nn.functional.conv1d(torch.nn.functional.pad(x.T[None], (2, 0)), w[:, None], groups=4)[0].T
    assert (O.short_conv(x, w) - want).abs().max() < 1e-12


def test_latent_attention_in_the_latent_space_is_the_same():
    """scores q W_uk . c and outputs W_uv (sum p c): what a decode step computes"""
    cfg, w = CONFIGS["wide"], {k: v.double() for k, v in weights("wide").items()}
    mx, p = cfg["layers"][1]["mixer"], "l1.mix."
    h = torch.randn(50, cfg["width"], dtype=torch.float64)
    want = O.latent_attention(h, w, p, mx, 1e-5)
    c = O.rms_norm(h @ w[p + "dkv"].T, w[p + "dkv.norm"], 1e-5)
    q = (O.rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], 1e-5) @ w[p + "uq"].T).view(50, mx["heads"], -1)
    ql = torch.einsum("thd,hdr->thr", q, w[p + "uk"].view(mx["heads"], mx["dim"], -1))
    s = torch.einsum("thr,jr->htj", ql, c) * mx["scale"]
    pr = s.masked_fill(~O.window_mask(50, mx["mask"]["size"]), float("-inf")).softmax(-1)
    o = torch.einsum("hvr,htr->thv", w[p + "uv"].view(mx["heads"], mx["vdim"], -1), torch.einsum("htj,jr->htr", pr, c))
    assert (o.reshape(50, -1) @ w[p + "o"].T - want).abs().max() < 1e-10


def test_router_keeps_the_largest():
    w = {"m.router": torch.eye(4, dtype=torch.float64), "m.router.b": torch.tensor([0.0, 0.0, 5.0, 0.0], dtype=torch.float64)}
    idx, wt = O.route(torch.tensor([[3.0, 1.0, 0.0, 2.0]], dtype=torch.float64), w, "m.", 2)
    assert idx.tolist() == [[2, 0]] and (wt[0] - torch.tensor([5.0, 3.0], dtype=torch.float64).softmax(0)).abs().max() < 1e-12


@pytest.mark.parametrize("name", list(CONFIGS))
def test_steady_routing_is_far_from_ties_and_varies(name, monkeypatch):
    gaps, picks = [], set()
    plain = O.route

    def spy(h, w, p, top):
        z = h @ w[p + "router"].T + w[p + "router.b"]
        if top < z.shape[1]:
            v = z.topk(top + 1, -1).values
            gaps.append((v[:, top - 1] - v[:, top]).min().item())
        idx, wt = plain(h, w, p, top)
        picks.update(tuple(r) for r in idx.tolist())
        return idx, wt
    monkeypatch.setattr(O, "route", spy)
    O.logits(CONFIGS[name], weights(name, steady=True), tokens(name, 200))
    assert all(g > 0.1 for g in gaps), min(gaps)
    if name in ("mixed", "plain", "wide"):
        assert len(picks) > 3


@pytest.mark.parametrize("what", ["window", "bigram", "loop", "conv", "decay", "top", "scale"])
def test_a_planted_mistake_shows(what):
    cfg, w, t = CONFIGS["mixed"], weights("mixed"), tokens("mixed", 60)
    want = O.logits(cfg, w, t)
    bad, wb = copy.deepcopy(cfg), dict(w)
    if what == "window":
        bad["layers"][1]["mixer"]["mask"]["size"] -= 1
    elif what == "bigram":
        bad["embedding"]["bigram"]["mul_prev"] += 1
    elif what == "loop":
        bad["loop"]["times"] -= 1
    elif what == "conv":
        wb["l0.mix.k.conv"] = w["l0.mix.k.conv"].flip(1)
    elif what == "decay":
        wb["l2.mix.dt_bias"] = w["l2.mix.dt_bias"] + 0.1
    elif what == "top":
        bad["layers"][2]["mlp"]["router"]["top"] = 2
    else:
        bad["layers"][3]["mixer"]["scale"] *= 1.05
    err = (O.logits(bad, wb, t) - want).pow(2).mean(-1).sqrt().max() / want.pow(2).mean().sqrt()
    assert err > 2e-3, err
