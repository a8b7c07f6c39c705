"""Plain, slow forward pass of the Siterax decoder (torch on the CPU, one function per mechanism, whole sequences only: no cache, no batching, no padding).

Test infrastructure: it shares no code with the engine and is compared with it by tests/test_siterax_*.py.  Everything is computed in `ft`
(float64 by default) from the weights as they are stored; x rows are [T, width] of one sequence, positions are 0 .. T-1.

    logits(cfg, w, tokens)          [T, vocab]
    residual_trace(cfg, w, tokens)  the residual stream after every layer run (a looped layer counts once per pass)
    greedy(cfg, w, tokens, n)       n greedy tokens by re-running the whole sequence
"""
from __future__ import annotations

import torch


def rms_norm(x, weight, eps):
    """x / sqrt(mean(x^2) + eps), times an elementwise weight when there is one (last dimension)."""
    y = x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def linear(x, w, bias=None):
    y = x @ w.T
    return y if bias is None else y + bias


def silu(z):
    return z * torch.sigmoid(z)


def rope_frequencies(rot, ft):
    """Angle per position of every pair: base^(-2 i / dims), divided by the linear scaling factor."""
    half = rot["dims"] // 2
    f = float(rot["base"]) ** (-2.0 * torch.arange(half, dtype=ft) / rot["dims"])
    return f / float((rot.get("scaling") or {}).get("factor", 1.0))


def rotate(x, positions, rot):
    """Rotary positions on the first rot.dims dimensions of x [T, heads, dim]; dimension i pairs with i + dims / 2; the rest passes."""
    half = rot["dims"] // 2
    ang = positions.to(x.dtype)[:, None] * rope_frequencies(rot, x.dtype)[None, :]
    c, s = ang.cos()[:, None, :], ang.sin()[:, None, :]
    u, v, rest = x[..., :half], x[..., half:2 * half], x[..., 2 * half:]
    return torch.cat([u * c - v * s, v * c + u * s, rest], dim=-1)


def window_mask(T, size):
    """[T, T] bool: query i sees key j iff 0 <= i - j < size (size None: every earlier key)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    ok = j <= i
    return ok if size is None else ok & (i - j < size)


def softmax_plus_one(scores, mask):
    """exp(s_j) / (1 + sum exp(s)) over the visible keys (last dimension): the extra 1 is a key of score 0 that carries no value."""
    s = scores.masked_fill(~mask, float("-inf"))
    m = s.max(dim=-1, keepdim=True).values.clamp_min(0.0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(dim=-1, keepdim=True))


def attention(h, w, p, mx, eps):
    """One attention mixer over h [T, width]; w maps tensor names, p is the layer's prefix ('l3.mix.')."""
    T = h.shape[0]
    H, G, dk, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = linear(h, w[p + "q"], w[p + "q.b"]).view(T, H, dk)
    k = linear(h, w[p + "k"], w[p + "k.b"]).view(T, G, dk)
    v = linear(h, w[p + "v"], w[p + "v.b"]).view(T, G, dv)
    q, k = rms_norm(q, w[p + "q.norm"], eps), rms_norm(k, w[p + "k.norm"], eps)
    pos = torch.arange(T)
    q, k = rotate(q, pos, mx["rot"]), rotate(k, pos, mx["rot"])
    mask = window_mask(T, (mx.get("mask") or {}).get("size"))
    gate = torch.sigmoid(linear(h, w[p + "g"]))                     # [T, H]
    out = torch.empty(T, H, dv, dtype=h.dtype)
    for head in range(H):
        kvh = head // (H // G)
        prob = softmax_plus_one((q[:, head] @ k[:, kvh].T) * mx["scale"], mask)
        out[:, head] = (prob @ v[:, kvh]) * gate[:, head:head + 1]
    return linear(out.reshape(T, H * dv), w[p + "o"])


def feed_forward(h, w, p):
    return linear(silu(linear(h, w[p + "gate"])) * linear(h, w[p + "up"]), w[p + "down"])


def layer_runs(cfg):
    """[(layer index, adds the embedding output first)] in execution order."""
    n = len(cfg["layers"])
    lp = cfg.get("loop") or {"start": 0, "stop": 0, "times": 1}
    runs = [(i, False) for i in range(lp["start"])]
    for t in range(lp["times"]):
        runs += [(i, t > 0 and i == lp["start"]) for i in range(lp["start"], lp["stop"])]
    return runs + [(i, False) for i in range(lp["stop"], n)]


def _forward(cfg, w, tokens, ft):
    w = {k: v.to(ft) for k, v in w.items()}
    eps, m = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])
    x0 = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    x, trace = x0, []
    for i, inject in layer_runs(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        if inject:
            x = x + x0
        x = x + m * rms_norm(attention(rms_norm(x, w[p + "norm1"], eps), w, p + "mix.", L["mixer"], eps), w[p + "norm1b"], eps)
        if L.get("mlp") is not None:
            x = x + m * rms_norm(feed_forward(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp."), w[p + "norm2b"], eps)
        trace.append(x)
    z = linear(rms_norm(x, w["final.norm"], eps), w["head"])
    cap = cfg.get("logit_softcap")
    return (z if cap is None else cap * torch.tanh(z / cap)), torch.stack(trace)


def logits(cfg, w, tokens, ft=torch.float64):
    return _forward(cfg, w, tokens, ft)[0]


def residual_trace(cfg, w, tokens, ft=torch.float64):
    return _forward(cfg, w, tokens, ft)[1]


def greedy(cfg, w, tokens, n, ft=torch.float64):
    seq = [int(t) for t in tokens]
    for _ in range(n):
        seq.append(int(logits(cfg, w, seq, ft)[-1].argmax()))
    return seq[len(tokens):]


def make_weights(cfg, seed=0, gain=1.0):
    """Random bfloat16 weights of a configuration: {tensor name: tensor}, names and shapes as a checkpoint of the design stores them."""
    g = torch.Generator().manual_seed(seed)
    rnd = lambda *s: torch.randn(*s, generator=g)
    D = cfg["width"]
    w = {"embed": rnd(cfg["vocab"], D)}
    for i, L in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", L["mixer"]
        H, G, dk, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
        norms = ["norm1", "norm1b"] + (["norm2", "norm2b"] if L.get("mlp") is not None else [])
        for nm in norms:
            w[p + nm] = 1 + 0.3 * rnd(D)
        for nm, n in (("q", H * dk), ("k", G * dk), ("v", G * dv)):
            w[p + "mix." + nm] = gain * rnd(n, D) / D ** 0.5
            w[p + f"mix.{nm}.b"] = 0.5 * rnd(n)
        w[p + "mix.q.norm"], w[p + "mix.k.norm"] = 1 + 0.3 * rnd(dk), 1 + 0.3 * rnd(dk)
        w[p + "mix.g"] = rnd(H, D) / D ** 0.5
        w[p + "mix.o"] = rnd(D, H * dv) / (H * dv) ** 0.5
        if L.get("mlp") is not None:
            ff = L["mlp"]["ff"]
            w[p + "mlp.gate"], w[p + "mlp.up"] = rnd(ff, D) / D ** 0.5, rnd(ff, D) / D ** 0.5
            w[p + "mlp.down"] = rnd(D, ff) / ff ** 0.5
    w["final.norm"] = 1 + 0.3 * rnd(D)
    w["head"] = rnd(cfg["vocab"], D) / D ** 0.5
    return {k: v.to(torch.bfloat16) for k, v in w.items()}
