"""Vizosun on the engine against the oracle: whole prompts, portions, token-by-token decoding, batches, reused sequences, long decoding, generation through every entry point
(generate, offline batch, scheduler, beams, command line, trace replay).  fp32 is compared tightly, 16 bits within rounding."""
import json
import os
import subprocess
import sys
import threading

import numpy as np
import pytest
import torch

from oracle import vizosun_oracle as O
from vizosun_util import CONFIGS, build, build_config, config, delta, dense, latent, moe, rel, save_checkpoint, tokens, weights

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DT = {"f32": torch.float32, "bf16": torch.bfloat16, "f16": torch.float16}
TOL = {"f32": 2e-5, "bf16": 4e-2, "f16": 6e-3}
NAMES = list(CONFIGS)
_m, _o = {}, {}


def model(name, dt):
    if (name, dt) not in _m:
        _m[name, dt] = build(name, DT[dt])
    return _m[name, dt]


def oracle(name, toks, dt="f32"):
    """logits for the weights `model(name, dt)` has (16-bit models: routing far from ties)"""
    steady = dt != "f32"
    key = (name, tuple(toks), steady)
    if key not in _o:
        _o[key] = O.logits(CONFIGS[name], weights(name, steady=steady), toks)
    return _o[key]


def run(m, toks, cuts=(), chunk=0):
    """logits of every position, the sequence brought in the given portions"""
    t = torch.tensor([toks], device=m.device)
    out, cache, a = [], None, 0
    for b in list(cuts) + [len(toks)]:
        if cache is None:
            r = m.forward(t[:, a:b], chunk=chunk)
            cache = r.past_key_values
        else:
            r = m.forward(t[:, a:b], past_key_values=cache, chunk=chunk)
        out.append(r.logits[0])
        a = b
    torch.cuda.synchronize()
    cache.close()
    return torch.cat(out)


@pytest.mark.parametrize("dt", list(DT))
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompts(cuda, name, dt):
    m = model(name, dt)
    for n in (1, 2, 7, 65, 300):
        t = tokens(name, n, n)
        assert rel(run(m, t), oracle(name, t, dt)) < TOL[dt], n


@pytest.mark.parametrize("name", NAMES)
def test_residual_stream_after_every_run(cuda, name):
    m, t = model(name, "f32"), tokens(name, 40)
    r = m.forward(torch.tensor([t], device=cuda), output_hidden_states=True)
    want = O.residual_trace(CONFIGS[name], weights(name), t)
    assert r.hidden_states.shape[0] == want.shape[0]
    for i in range(want.shape[0]):
        assert rel(r.hidden_states[i, 0], want[i]) < TOL["f32"], i
    assert rel(r.logits[0], oracle(name, t)) < TOL["f32"]
    # pieces of the same prompt leave the same trace-free logits
    assert rel(run(m, t, chunk=16), oracle(name, t)) < TOL["f32"]


@pytest.mark.parametrize("dt", list(DT))
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("cuts", [(2,), (1, 3), (63, 64), (65, 127, 129), (24, 25, 48), (16, 32, 33), tuple(range(2, 140, 2)), (17, 40, 90)])
def test_portions_of_a_prompt(cuda, name, dt, cuts):
    t = tokens(name, 140)
    assert rel(run(model(name, dt), t, cuts), oracle(name, t, dt)) < TOL[dt]


@pytest.mark.parametrize("dt", list(DT))
@pytest.mark.parametrize("name", NAMES)
def test_token_by_token_from_the_first(cuda, name, dt):
    """every window is passed by decoded tokens; page and chunk borders are crossed"""
    t = tokens(name, 270)
    got = run(model(name, dt), t, tuple(range(1, 270)))
    assert rel(got, oracle(name, t, dt)) < TOL[dt]


@pytest.mark.parametrize("dt", ["f32", "bf16"])
@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_decode_after_a_prompt(cuda, name, dt):
    t = tokens(name, 200, 3)
    for p in (23, 24, 25, 63, 64, 65, 127, 128, 129, 131):
        got = run(model(name, dt), t[:p + 6], tuple(range(p, p + 6)))
        assert rel(got, oracle(name, t, dt)[:p + 6]) < TOL[dt], p


def _batch_logits(m, prompts, extra):
    """prompts prefilled together, then decoded together; returns all logits per request (prompt rows and decoded rows)"""
    from llava_mi355x.batching import DecodeBatch
    from llava_mi355x.engine_lm import LmxKVCache
    caches = [LmxKVCache(m, 1) for _ in prompts]
    emb = [m.get_model().embed_tokens(torch.tensor(p)) for p in prompts]
    lg = m.prefill_logits(caches, emb, [list(range(len(p))) for p in prompts])
    rows = [list(r) for r in lg.split([len(p) for p in prompts])]
    live = list(range(len(prompts)))
    b = DecodeBatch(m, len(prompts))
    for s in range(max(len(e) for e in extra)):
        live = [i for i in live if s < len(extra[i])]
        out = torch.empty((len(live), m._vocab_cap), dtype=m.logits_dtype, device=m.device)
        b.step([caches[i].seqs[0] for i in live], [extra[i][s] for i in live], 1, False, out)
        for i, r in zip(live, out):
            rows[i].append(r.clone())
    torch.cuda.synchronize()
    b.close()
    for c in caches:
        c.close()
    return [torch.stack(r)[:, : m.config.vocab_size] for r in rows]


@pytest.mark.parametrize("dt", list(DT))
@pytest.mark.parametrize("name", NAMES)
def test_batches_of_unequal_requests(cuda, name, dt):
    lens, dec = [1, 130, 40, 65, 7], [9, 3, 5, 0, 12]
    ts = [tokens(name, n + d, 20 + i) for i, (n, d) in enumerate(zip(lens, dec))]
    got = _batch_logits(model(name, dt), [t[:n] for t, n in zip(ts, lens)], [t[n:] for t, n in zip(ts, lens)])
    for t, g in zip(ts, got):
        assert rel(g, oracle(name, t, dt)) < TOL[dt]
    if dt != "f32":                                     # alone: equal up to rounding
        alone = run(model(name, dt), ts[1], tuple(range(lens[1], len(ts[1]))))
        assert rel(got[1], alone.double().cpu()) < TOL[dt]


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_many_sequences_in_one_decode_batch(cuda, dt):
    """more rows than the decode-batch kernel takes"""
    ts = [tokens("mixed", 5 + i % 7, 60 + i) for i in range(40)]
    got = _batch_logits(model("mixed", dt), [t[:-2] for t in ts], [t[-2:] for t in ts])
    assert max(rel(g, oracle("mixed", t, dt)) for g, t in zip(got, ts)) < TOL[dt]


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_sequences_that_are_freed_and_used_again(cuda, dt):
    m = model("mixed", dt)
    t1, t2 = tokens("mixed", 200, 1), tokens("mixed", 30, 2)
    first = run(m, t2, tuple(range(20, 30)))
    for _ in range(3):
        run(m, t1, (100,))                              # fills the pooled sequence's rows well past the next request's
        again = run(m, t2, tuple(range(20, 30)))
        assert torch.equal(first, again)


def test_sequences_with_state_are_cut_to_nothing_or_not_at_all(cuda):
    from llava_mi355x._C import check, lib, stream_handle
    m, t = model("mixed", "f32"), tokens("mixed", 120, 4)
    c = m.forward(torch.tensor([t], device=cuda)).past_key_values
    assert lib.lmx_seq_truncate(c.seqs[0], 50, stream_handle()) != 0 and lib.lmx_seq_length(c.seqs[0]) == 120
    check(lib.lmx_seq_truncate(c.seqs[0], 120, stream_handle()), "truncate")
    more = tokens("mixed", 9, 9)
    got = m.forward(torch.tensor([more], device=cuda), past_key_values=c).logits[0]
    assert rel(got, oracle("mixed", t + more)[120:]) < TOL["f32"]
    check(lib.lmx_seq_truncate(c.seqs[0], 0, stream_handle()), "truncate")
    got = m.forward(torch.tensor([more], device=cuda), past_key_values=c).logits[0]      # a new sequence in the old one's memory
    assert rel(got, oracle("mixed", more)) < TOL["f32"]
    c.close()


def test_copied_sequences_carry_state_and_previous_token(cuda):
    from llava_mi355x._C import check, lib, stream_handle
    from llava_mi355x.engine_lm import LmxKVCache
    m, t = model("mixed", "f32"), tokens("mixed", 60, 14)
    a = m.forward(torch.tensor([t], device=cuda)).past_key_values
    b = LmxKVCache(m, 1)
    check(lib.lmx_seq_copy(b.seqs[0], a.seqs[0], stream_handle()), "seq_copy")
    for c, more in ((a, tokens("mixed", 5, 1)), (b, tokens("mixed", 7, 2))):
        got = torch.cat([m.forward(torch.tensor([[x]], device=cuda), past_key_values=c).logits[0] for x in more])
        assert rel(got, oracle("mixed", t + more)[60:]) < TOL["f32"]
    a.close(); b.close()


def test_window_edges_in_the_model(cuda):
    """two sequences that differ in one token at distances inside, at the edge of and outside a window; prompt and decoded.  Without a bigram table and recurrent layers a
    key outside the window cannot move anything"""
    cfg = config([latent(2, 50, 66, 70, 20, 65, dense(33), scale=2.0)], 100, 97, None, bigram=None)
    w = O.make_weights(cfg, 5)
    m = build_config(cfg, w, torch.float32)
    base = tokens("odd", 260, 8)
    for dist in (1, 63, 64, 65, 66, 128, 200):
        a, b = list(base), list(base)
        a[255 - dist], b[255 - dist] = 11, 45
        for cuts in ((), (250,) + tuple(range(251, 260)), (192, 254)):
            ga, gb = run(m, a, cuts), run(m, b, cuts)
            assert rel(ga, O.logits(cfg, w, a)) < TOL["f32"] and rel(gb, O.logits(cfg, w, b)) < TOL["f32"]
            moved = (ga[255] - gb[255]).abs().max().item()
            assert (moved > 2e-6) if dist <= 64 else moved == 0, (dist, cuts, moved)


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_a_far_token_stays_in_the_state(cuda, dt):
    """slow decays: the first tokens move the logits hundreds of positions later, through portions and through decoding alike"""
    cfg = config([delta(2, 1, 40, 24, 4, dense(40)), delta(3, 3, 72, 40, 3, None)], 100, 97, None, bigram=None)
    w = O.make_weights(cfg, 6)
    for k in w:
        if k.endswith("dt_bias"):
            w[k] = w[k] - 6.0
    m = build_config(cfg, w, DT[dt])
    a = tokens("odd", 330, 3)
    b = [(a[0] + 40) % 97, (a[1] + 3) % 97] + a[2:]
    wa, wb = O.logits(cfg, w, a), O.logits(cfg, w, b)
    assert (wa - wb)[300:].pow(2).mean(-1).sqrt().min() > 1e-3 * wa.pow(2).mean().sqrt()
    for cuts in ((), (2,), (100, 101, 300), (290,) + tuple(range(291, 330))):
        assert rel(run(m, a, cuts), wa) < TOL[dt] and rel(run(m, b, cuts), wb) < TOL[dt]
        if dt == "f32":
            assert rel((run(m, a, cuts) - run(m, b, cuts))[300:], (wa - wb)[300:]) < 2e-2


@pytest.mark.parametrize("a_log,dt_bias", [(4.0, 4.0), (-9.0, -6.0), (1.0, 0.0)])
def test_decays_of_any_strength(cuda, a_log, dt_bias):
    """states that vanish within a token, that keep everything, and both next to each other in one head: prompts (in chunks), portions across their borders, decoding"""
    cfg = config([delta(3, 1, 70, 40, 3, None), delta(2, 2, 64, 130, 4, dense(40))], 96, 80)
    w = O.make_weights(cfg, 5, (33, 20))
    for i in (0, 1):
        w[f"l{i}.mix.A_log"] = torch.full_like(w[f"l{i}.mix.A_log"], a_log)
        b = torch.full_like(w[f"l{i}.mix.dt_bias"], dt_bias)
        b[::5] = -dt_bias
        w[f"l{i}.mix.dt_bias"] = b
    m, t = build_config(cfg, w, torch.float32), torch.randint(0, 80, (150,), generator=torch.Generator().manual_seed(3)).tolist()
    want = O.logits(cfg, w, t)
    for cuts in ((), (15, 16, 17, 31, 33, 64), (20,) + tuple(range(140, 150))):
        got = run(m, t, cuts)
        assert torch.isfinite(got).all() and rel(got, want) < TOL["f32"], cuts


def test_the_first_tokens_of_a_sequence(cuda):
    """the row without a previous token, and convolutions that reach before the start; the second token looks back at the first, however it arrives"""
    for name in ("mixed", "odd", "wide"):
        m = model(name, "f32")
        for n in (1, 2, 3, 5, 6):
            t = tokens(name, n, 40 + n)
            for cuts in ((), tuple(range(1, n)), (n - 1,) if n > 1 else ()):
                assert rel(run(m, t, cuts), oracle(name, t)) < TOL["f32"], (name, n, cuts)


def test_a_stopped_sequence_keeps_its_state(cuda):
    """steps queued past a device-side stop leave state, ring and previous token alone: the next turn continues the finished one"""
    m, p = build("mixed", torch.float32), tokens("mixed", 40, 6)
    ids = O.greedy(CONFIGS["mixed"], weights("mixed"), p, 12)
    eos = ids[4]
    cut = ids[: ids.index(eos) + 1]
    m.enable_reuse(images=0, prefixes=4, min_rows=8)
    out = m.generate(torch.tensor([p], device=cuda), max_new_tokens=12, eos_token_id=eos, run_ahead=8)[0].tolist()
    assert out == p + cut
    longer = out + tokens("mixed", 5, 3)
    b = m.generate(torch.tensor([longer], device=cuda), max_new_tokens=6, eos_token_id=-1)[0, len(longer):].tolist()
    assert m.reuse_stats()["prefix_hits"] == 1 and b == O.greedy(CONFIGS["mixed"], weights("mixed"), longer, 6)
    other = out[:30] + tokens("mixed", 9, 4)                      # another way after 30 rows: nothing to reuse
    b = m.generate(torch.tensor([other], device=cuda), max_new_tokens=6, eos_token_id=-1)[0, len(other):].tolist()
    assert m.reuse_stats()["prefix_hits"] == 1 and b == O.greedy(CONFIGS["mixed"], weights("mixed"), other, 6)
    m.disable_reuse()


@pytest.mark.parametrize("dt", ["f32", "bf16"])
def test_long_decoding(cuda, dt):
    """greedy ids fed back for many steps: the logits along the way stay the oracle's for the same ids"""
    m = model("mixed", dt)
    p = tokens("mixed", 9, 5)
    out = m.generate(torch.tensor([p], device=cuda), max_new_tokens=400, eos_token_id=-1)[0].tolist()
    assert len(out) == 409
    want = oracle("mixed", out[:-1], dt)
    got = run(m, out[:-1], tuple(range(9, 408)))
    assert rel(got, want) < TOL[dt]
    if dt == "f32":
        margin = want[8:].topk(2, -1).values
        sure = (margin[:, 0] - margin[:, 1]) > 1e-3
        assert torch.equal(want[8:].argmax(-1)[sure], torch.tensor(out[9:])[sure])


@pytest.mark.parametrize("name", NAMES)
def test_greedy_generation_is_the_oracles(cuda, name):
    m = model(name, "f32")
    for n in (1, 30):
        p = tokens(name, n, 6)
        want = O.greedy(CONFIGS[name], weights(name), p, 20)
        assert m.generate(torch.tensor([p], device=cuda), max_new_tokens=20, eos_token_id=-1)[0, n:].tolist() == want
        eos = want[7]
        cut = want[: want.index(eos) + 1]
        assert m.generate(torch.tensor([p], device=cuda), max_new_tokens=20, eos_token_id=eos)[0, n:].tolist() == cut


def test_offline_batch_scheduler_and_prefix_reuse(cuda):
    m = build("mixed", torch.float32)
    ps = [tokens("mixed", n, 70 + n) for n in (3, 50, 17, 1, 90, 33)]
    want = [O.greedy(CONFIGS["mixed"], weights("mixed"), p, 12) for p in ps]
    outs = m.generate_batch([torch.tensor(p) for p in ps], max_new_tokens=12, eos_token_id=-1)
    assert [o[len(p):].tolist() for o, p in zip(outs, ps)] == want
    m.enable_batching(capacity=4)
    try:
        got = [None] * len(ps)

        def work(i):
            got[i] = m.generate(torch.tensor([ps[i]], device=cuda), max_new_tokens=12, eos_token_id=-1)[0, len(ps[i]):].tolist()
        th = [threading.Thread(target=work, args=(i,)) for i in range(len(ps))]
        [t.start() for t in th]; [t.join(60) for t in th]
        assert got == want
        assert m._batcher.prefilled == len(ps)
    finally:
        m.disable_batching()
    m.enable_reuse(images=0, prefixes=4, min_rows=8)
    a = m.generate(torch.tensor([ps[4]], device=cuda), max_new_tokens=12, eos_token_id=-1)[0].tolist()
    longer = a + tokens("mixed", 5, 3)
    b = m.generate(torch.tensor([longer], device=cuda), max_new_tokens=6, eos_token_id=-1)[0, len(longer):].tolist()
    assert m.reuse_stats()["prefix_hits"] == 1 and b == O.greedy(CONFIGS["mixed"], weights("mixed"), longer, 6)
    m.disable_reuse()


def test_sampling_follows_the_logits(cuda):
    m = model("single", "bf16")
    p = torch.tensor([tokens("single", 12, 1)], device=cuda)
    torch.manual_seed(0)
    a = m.generate(p, max_new_tokens=16, do_sample=True, temperature=0.9, top_p=0.9, eos_token_id=-1).tolist()
    torch.manual_seed(0)
    assert a == m.generate(p, max_new_tokens=16, do_sample=True, temperature=0.9, top_p=0.9, eos_token_id=-1).tolist()
    torch.manual_seed(1)
    assert a != m.generate(p, max_new_tokens=16, do_sample=True, temperature=0.9, top_p=0.9, eos_token_id=-1).tolist()
    greedy = m.generate(p, max_new_tokens=16, eos_token_id=-1).tolist()
    assert greedy == m.generate(p, max_new_tokens=16, do_sample=True, temperature=0.9, top_k=1, eos_token_id=-1).tolist()


def test_beam_search_is_at_least_greedy(cuda):
    m, p = model("mixed", "f32"), tokens("mixed", 10, 2)

    def score(new):
        lp = O.logits(CONFIGS["mixed"], weights("mixed"), p + new).log_softmax(-1)
        return sum(lp[len(p) - 1 + i, t].item() for i, t in enumerate(new))
    beam = m.generate(torch.tensor([p], device=cuda), max_new_tokens=6, num_beams=4, eos_token_id=-1)[0, 10:].tolist()
    greedy = O.greedy(CONFIGS["mixed"], weights("mixed"), p, 6)
    assert len(beam) == 6 and score(beam) >= score(greedy) - 1e-4


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_fused_and_separate_decode_launches_agree(cuda, name):
    m, t = model(name, "bf16"), tokens(name, 60)
    cuts = tuple(range(30, 60))
    a = run(m, t, cuts)
    m.set_option("stack_fuse", 0)
    try:
        b = run(m, t, cuts)
    finally:
        m.set_option("stack_fuse", 1)
    assert rel(a, b.double().cpu()) < TOL["bf16"] / 2


def test_loading_checks_names_and_shapes(cuda):
    from llava_mi355x._C import LmxError
    from llava_mi355x.vizosun import VizosunConfig, VizosunForCausalLM
    w = weights("mixed")
    mk = lambda: VizosunForCausalLM(VizosunConfig.from_dict(CONFIGS["mixed"], {k: tuple(v.shape) for k, v in w.items()}), dtype=torch.bfloat16, max_position=128)
    m = mk()
    for k in ("l0.mix.v.conv", "final.norm", "bigram", "loop.in", "l1.mlp.e3.up", "l2.mlp.router.b", "l3.mix.dkv.norm"):
        with pytest.raises(LmxError, match="missing tensors: .*" + k.replace(".", r"\.")):
            mk().load_state_dict({n: t for n, t in w.items() if n != k})
    for k in ("l1.mix.uk", "l0.mix.a2", "l2.mlp.e1.down", "l0.mix.q.conv"):
        with pytest.raises(LmxError, match="shape mismatch"):
            m.load_tensor(k, w[k].T)
    for k in ("l0.mix.z", "l0.norm2", "l1.mlp.gate", "l1.mlp.e5.up", "l0.mlp.e0.up", "head", "l3.mix.q"):
        with pytest.raises(LmxError, match="unknown tensor|out of range|shape"):
            m.load_tensor(k, w["embed"])
    with pytest.raises(LmxError, match="capacity"):
        m.load_state_dict(w).forward(torch.tensor([[1] * 129], device=cuda))


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_trace_replay(cuda, tmp_path, dt):
    cfg, w = CONFIGS["mixed"], weights("mixed", steady=dt != "float32")
    save_checkpoint(str(tmp_path / "m"), cfg, w)
    ts = {"x": tokens("mixed", 70, 1), "y": tokens("mixed", 9, 2), "z": tokens("mixed", 33, 3)}
    feed = [[("x", 60), ("y", 3), ("z", 30)], [("x", 1), ("y", 1), ("z", 1)], [("x", 9), ("y", 5), ("z", 2)]]
    at, lines, keys = dict.fromkeys(ts, 0), [], []
    for s, step in enumerate(feed):
        ent = []
        for r, n in step:
            want = sorted({0, n // 2, n - 1}) if not (s == 1 and r == "y") else []
            ent.append({"id": r, "tokens": ts[r][at[r]:at[r] + n], "want": want})
            keys += [(s, r, at[r] + k) for k in want]
            at[r] += n
        lines.append({"step": s, "entries": ent, "end": ["x", "y", "z"] if s == 2 else []})
    lines.append({"step": 7, "entries": [{"id": "x", "tokens": ts["y"], "want": []}], "end": ["x"]})
    os.makedirs(tmp_path / "o")
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", dt, "--out", str(tmp_path / "o"), "--max-tokens", "256"],
                       input="".join(json.dumps(x) + "\n" for x in lines), capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2", "done 7"]
    assert sorted(os.listdir(tmp_path / "o")) == ["0.f32", "1.f32", "2.f32"]
    got = np.concatenate([np.fromfile(tmp_path / "o" / f"{s}.f32", dtype="<f4").reshape(-1, cfg["vocab"]) for s in range(3)])
    want = torch.stack([oracle("mixed", ts[q], "f32" if dt == "float32" else "bf16")[p] for _, q, p in keys])
    assert rel(torch.from_numpy(got), want) < TOL["f32" if dt == "float32" else "bf16"]


def test_generation_command_line(cuda, tmp_path):
    save_checkpoint(str(tmp_path), CONFIGS["odd"], weights("odd"))
    ps = [tokens("odd", 5, 1), tokens("odd", 12, 2)]
    env = dict(os.environ, PYTHONPATH=os.path.join(ROOT, "llava-plus-codebase_amd"))
    r = subprocess.run([sys.executable, "-m", "llava_mi355x.cli", "--model", str(tmp_path), "--dtype", "float32", "--max-new-tokens", "8", "--max-position", "128"]
                       + [x for p in ps for x in ("--tokens", ",".join(map(str, p)))], capture_output=True, text=True, timeout=110, env=env)
    assert r.returncode == 0, r.stderr[-2000:]
    want = [O.greedy(CONFIGS["odd"], weights("odd"), p, 8) for p in ps]
    assert [[int(t) for t in x.split(",")] for x in r.stdout.split()] == want


def test_load_pretrained_model_serves_the_family(cuda, tmp_path):
    from llava_mi355x.builder import load_pretrained_model
    save_checkpoint(str(tmp_path), CONFIGS["odd"], weights("odd"))
    tok, m, proc, ctx = load_pretrained_model(str(tmp_path), None, "vizosun-test", torch_dtype=torch.float32, max_position=128)
    assert tok is None and proc is None and ctx == 128
    p = tokens("odd", 6, 4)
    assert m.generate(torch.tensor([p], device=cuda), max_new_tokens=5, eos_token_id=-1)[0, 6:].tolist() == O.greedy(CONFIGS["odd"], weights("odd"), p, 5)
