"""Plain, slow forward pass of the Vizosun decoder (torch on the CPU, one function per mechanism, whole sequences only: no cache, no batching, no padding).

Test infrastructure: it shares no code with the engine and is compared with it by tests/test_vizosun_*.py.  Everything is computed in `ft`
(float64 by default) from the weights as they are stored; x rows are [T, width] of one sequence, positions are 0 .. T-1.

    logits(cfg, w, tokens)          [T, vocab]
    residual_trace(cfg, w, tokens)  the residual stream after every layer run (a looped layer counts once per pass)
    greedy(cfg, w, tokens, n)       n greedy tokens by re-running the whole sequence
"""
from __future__ import annotations

import torch


def rms_norm(x, weight, eps):
    """x / sqrt(mean(x^2) + eps) over the last dimension, times an elementwise weight when there is one."""
    y = x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def linear(x, w):
    return x @ w.T


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(z.clamp(max=30))))


def bigram_rows(tokens, bg):
    """Row of the bigram table for every position: a hash of (previous token, token); the extra last row where there is no previous token."""
    rows, prev = [], None
    for t in tokens:
        t = int(t)
        rows.append(bg["buckets"] if prev is None else (prev * bg["mul_prev"] + t * bg["mul_cur"]) % bg["buckets"])
        prev = t
    return rows


def embedding(cfg, w, tokens):
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    bg = (cfg.get("embedding") or {}).get("bigram")
    return x if not bg else x + w["bigram"][torch.as_tensor(bigram_rows(tokens, bg), dtype=torch.long)]


def window_mask(T, size):
    """[T, T] bool: query i sees key j iff 0 <= i - j < size (size None: every earlier key)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    ok = j <= i
    return ok if size is None else ok & (i - j < size)


def latent_attention(h, w, p, mx, eps):
    """Queries and keys / values through low-rank latents, no positions, softmax over a window."""
    T = h.shape[0]
    H, dk, dv = mx["heads"], mx["dim"], mx["vdim"]
    cq = rms_norm(linear(h, w[p + "dq"]), w[p + "dq.norm"], eps)
    c = rms_norm(linear(h, w[p + "dkv"]), w[p + "dkv.norm"], eps)
    q = linear(cq, w[p + "uq"]).view(T, H, dk)
    k = linear(c, w[p + "uk"]).view(T, H, dk)
    v = linear(c, w[p + "uv"]).view(T, H, dv)
    mask = window_mask(T, (mx.get("mask") or {}).get("size"))
    out = torch.empty(T, H, dv, dtype=h.dtype)
    for head in range(H):
        s = (q[:, head] @ k[:, head].T) * mx["scale"]
        out[:, head] = torch.softmax(s.masked_fill(~mask, float("-inf")), dim=-1) @ v[:, head]
    return linear(out.reshape(T, H * dv), w[p + "o"])


def short_conv(x, taps):
    """Causal convolution over time, one filter per channel: x [T, C], taps [C, n]; the last tap multiplies the current row, rows before the first are zero."""
    T, n = x.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, x.shape[1], dtype=x.dtype), x])
    return sum(padded[j:j + T] * taps[:, j] for j in range(n))


def unit(x):
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, g, beta):
    """Gated delta rule with a decay per key channel, token by token: q, k, g [T, H, dk], v [T, H, dv], beta [T, H] -> o [T, H, dv]."""
    T, H, dk = k.shape
    S = torch.zeros(H, dk, v.shape[2], dtype=k.dtype)
    out = []
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hkv,hk->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append(torch.einsum("hkv,hk->hv", S, q[t]))
    return torch.stack(out)


def decays(h, w, p, H, dk):
    """exp(-exp(A_log) softplus(W_a2 W_a1 h + dt_bias)), [T, H, dk]"""
    z = softplus(linear(linear(h, w[p + "a1"]), w[p + "a2"]) + w[p + "dt_bias"]).view(-1, H, dk)
    return torch.exp(-torch.exp(w[p + "A_log"])[None, :, None] * z)


def channel_delta(h, w, p, mx, eps):
    T = h.shape[0]
    H, G, dk, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q, k, v = (silu(short_conv(linear(h, w[p + n]), w[p + n + ".conv"])) for n in ("q", "k", "v"))
    q = (unit(q.view(T, G, dk)) * dk ** -0.5).repeat_interleave(H // G, dim=1)
    k = unit(k.view(T, G, dk)).repeat_interleave(H // G, dim=1)
    o = delta_rule(q, k, v.view(T, H, dv), decays(h, w, p, H, dk), torch.sigmoid(linear(h, w[p + "b"])))
    gate = torch.sigmoid(linear(linear(h, w[p + "g1"]), w[p + "g2"])).view(T, H, dv)
    return linear((rms_norm(o, w[p + "norm"], eps) * gate).reshape(T, H * dv), w[p + "o"])


def dense(h, w, p):
    return linear(torch.relu(linear(h, w[p + "gate"])) * linear(h, w[p + "up"]), w[p + "down"])


def route(h, w, p, top):
    """(chosen experts [T, top], their weights [T, top]): the largest router logits and the softmax over those alone."""
    z = linear(h, w[p + "router"]) + w[p + "router.b"]
    val, idx = z.topk(top, dim=-1)
    return idx, torch.softmax(val, dim=-1)


def mixture(h, w, p, mlp):
    idx, wt = route(h, w, p, mlp["router"]["top"])
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(idx[t].tolist(), wt[t]):
            x, q = h[t], p + f"e{e}."
            y[t] += a * (w[q + "down"] @ (silu(w[q + "gate"] @ x) * (w[q + "up"] @ x)))
    return y


MIXERS = {"latent_attention": latent_attention, "channel_delta": channel_delta}


def layer(x, w, i, L, eps):
    """Both sublayers read one norm: x + mixer(h) + ff(h)."""
    h = rms_norm(x, w[f"l{i}.norm1"], eps)
    y = MIXERS[L["type"]](h, w, f"l{i}.mix.", L["mixer"], eps)
    mlp = L.get("mlp")
    if mlp is not None:
        y = y + (dense(h, w, f"l{i}.mlp.") if mlp["kind"] == "dense" else mixture(h, w, f"l{i}.mlp.", mlp))
    return x + y


def layer_runs(cfg):
    """[(layer index, starts a pass of the loop)] in execution order."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    runs = [(i, False) for i in range(lp["start"])]
    for _ in range(lp["times"]):
        runs += [(i, i == lp["start"]) for i in range(lp["start"], lp["stop"])]
    return runs + [(i, False) for i in range(lp["stop"], n)]


def _forward(cfg, w, tokens, ft):
    w = {k: v.to(ft) for k, v in w.items()}
    eps = float(cfg["norm"]["eps"])
    x0 = embedding(cfg, w, tokens)
    x, trace = x0, []
    for i, begins in layer_runs(cfg):
        if begins:
            x = linear(torch.cat([x, x0], dim=-1), w["loop.in"])
        x = layer(x, w, i, cfg["layers"][i], eps)
        trace.append(x)
    return linear(rms_norm(x, w["final.norm"], eps), w["embed"]), torch.stack(trace)


def logits(cfg, w, tokens, ft=torch.float64):
    return _forward(cfg, w, tokens, ft)[0]


def residual_trace(cfg, w, tokens, ft=torch.float64):
    return _forward(cfg, w, tokens, ft)[1]


def greedy(cfg, w, tokens, n, ft=torch.float64):
    seq = [int(t) for t in tokens]
    for _ in range(n):
        seq.append(int(logits(cfg, w, seq, ft)[-1].argmax()))
    return seq[len(tokens):]


def make_weights(cfg, seed=0, ranks=(24, 20)):
    """Random bfloat16 weights of a configuration: {tensor name: tensor}, names and shapes as a checkpoint of the design stores them.  `ranks`: inner sizes of the decay
    and the output-gate projections (no configuration entry names them)."""
    g = torch.Generator().manual_seed(seed)
    rnd = lambda *s: torch.randn(*s, generator=g)
    mat = lambda n, k: rnd(n, k) / k ** 0.5
    D = cfg["width"]
    w = {"embed": rnd(cfg["vocab"], D) * 0.7}
    bg = (cfg.get("embedding") or {}).get("bigram")
    if bg:
        w["bigram"] = rnd(bg["buckets"] + 1, D) * 0.7
    if cfg.get("loop"):
        w["loop.in"] = mat(D, 2 * D)
    for i, L in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", L["mixer"]
        m = p + "mix."
        H, dk, dv = mx["heads"], mx["dim"], mx["vdim"]
        w[p + "norm1"] = 1 + 0.3 * rnd(D)
        if L["type"] == "latent_attention":
            R, Q = mx["kv_rank"], mx["q_rank"]
            w[m + "dq"], w[m + "uq"], w[m + "dkv"], w[m + "uk"], w[m + "uv"] = mat(Q, D), 1.5 * mat(H * dk, Q), mat(R, D), mat(H * dk, R), mat(H * dv, R)
            w[m + "dq.norm"], w[m + "dkv.norm"] = 1 + 0.3 * rnd(Q), 1 + 0.3 * rnd(R)
        else:
            G, n = mx["kv_heads"], mx["conv"]
            for nm, c in (("q", G * dk), ("k", G * dk), ("v", H * dv)):
                w[m + nm], w[m + nm + ".conv"] = 1.5 * mat(c, D), rnd(c, n) / n ** 0.5
            w[m + "b"], w[m + "A_log"], w[m + "dt_bias"], w[m + "norm"] = mat(H, D), rnd(H) - 1.0, rnd(H * dk) - 2.0, 1 + 0.3 * rnd(dv)
            w[m + "a1"], w[m + "a2"], w[m + "g1"], w[m + "g2"] = mat(ranks[0], D), mat(H * dk, ranks[0]), mat(ranks[1], D), mat(H * dv, ranks[1])
        w[m + "o"] = mat(D, H * dv)
        mlp = L.get("mlp")
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            ff = mlp["ff"]
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = mat(ff, D), mat(ff, D), mat(D, ff)
        else:
            ff, E = mlp["expert"]["ff"], mlp["router"]["experts"]
            for e in range(E):
                w[p + f"mlp.e{e}.gate"], w[p + f"mlp.e{e}.up"], w[p + f"mlp.e{e}.down"] = mat(ff, D), mat(ff, D), 2 * mat(D, ff)
            w[p + "mlp.router"], w[p + "mlp.router.b"] = 2 * mat(E, D), 0.5 * rnd(E)
    w["final.norm"] = 1 + 0.3 * rnd(D)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}
