"""Configurations and helpers of the Vizosun tests: small, unequal sizes on purpose (no two numbers of a layer are equal unless the case is about that)."""
import torch

from oracle import vizosun_oracle as O
from siterax_util import rel, save_checkpoint  # noqa: F401


def latent(heads, dim, vdim, q_rank, kv_rank, window, mlp, scale=None):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                                                  "scale": scale if scale is not None else 1.5 * dim ** -0.5, "mask": {"size": window} if window else None}, "mlp": mlp}


def delta(heads, kv_heads, dim, vdim, conv, mlp):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def config(layers, width, vocab, loop=None, bigram=(101, 7, 13), eps=1e-5):
    return {"architecture": "Vizosun", "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))} if bigram else {}, "layers": layers, "width": width, "vocab": vocab,
            "loop": loop, "norm": {"eps": eps}}


CONFIGS = {
    # every layer another shape, the loop in the middle
    "mixed": config([delta(4, 2, 24, 40, 3, dense(88)), latent(3, 40, 20, 50, 36, 24, moe(40, 5, 2)), delta(2, 1, 72, 33, 5, moe(72, 7, 3)), latent(5, 16, 80, 130, 70, 70, dense(33))],
                    136, 211, {"start": 1, "stop": 3, "times": 3}),
    # no loop; a window of one key, one tap, one expert of one, a layer without feed-forward; a bigram table larger than the vocabulary's pairs need
    "odd": config([delta(3, 3, 20, 12, 1, moe(24, 1, 1)), latent(2, 20, 12, 10, 9, 1, None), delta(1, 1, 64, 64, 2, None), latent(2, 50, 66, 70, 20, 65, dense(33))], 100, 97, None,
                  bigram=(1009, 211, 1), eps=1e-3),
    # no bigram table, the loop from the first layer to the last, latent attention over everything
    "plain": config([latent(4, 48, 48, 40, 60, 0, dense(100)), delta(4, 4, 48, 30, 4, moe(56, 6, 4))], 120, 90, {"start": 0, "stop": 2, "times": 2}, bigram=None),
    # head vectors and latents past 128
    "wide": config([delta(2, 1, 150, 200, 4, dense(70)), latent(2, 160, 136, 200, 300, 40, moe(50, 4, 2))], 128, 64, {"start": 0, "stop": 1, "times": 2}, bigram=(3, 5, 2)),
    # more heads than one workgroup takes, a latent past 128 seen from everywhere, more experts than most of the rows choose
    "many": config([latent(18, 24, 20, 44, 130, 0, moe(40, 21, 5)), delta(6, 3, 100, 70, 4, dense(64)), latent(3, 70, 72, 36, 257, 150, None)], 132, 150, {"start": 1, "stop": 3, "times": 2},
                   bigram=(67, 3, 11)),
    # one head, equal sizes, one pass
    "single": config([delta(1, 1, 128, 128, 4, dense(128)), latent(1, 128, 128, 128, 128, 128, moe(128, 2, 2))], 128, 128, {"start": 0, "stop": 2, "times": 1}, bigram=(128, 1, 1)),
}
RANKS = {"mixed": (18, 70), "odd": (7, 5), "plain": (64, 64), "wide": (130, 9), "single": (128, 128), "many": (65, 30)}


def steady_routing(cfg, w):
    """Weights whose router choices are far from ties in 16 bits and still differ from token to token: two stream dimensions carry two bits of the token id through all
    layers, the experts' logits follow them."""
    w = {k: v.clone() for k, v in w.items()}
    D, ids = cfg["width"], torch.arange(cfg["vocab"])
    for d in (0, 1):
        w["embed"][:, d] = 12.0 * (1 - 2 * ((ids >> d) & 1)).to(torch.bfloat16)
        if "bigram" in w:
            w["bigram"][:, d] = 0
        if "loop.in" in w:
            w["loop.in"][d] = 0
            w["loop.in"][d, D + d] = 1
        for k in w:
            if k.endswith((".o", ".down")):
                w[k][d] = 0
    for i, L in enumerate(cfg["layers"]):
        if (L.get("mlp") or {}).get("kind") == "moe":
            E = L["mlp"]["router"]["experts"]
            e = torch.arange(E)
            r = w[f"l{i}.mlp.router"]
            r *= 0.04
            for d in (0, 1):
                r[:, d] = 2.0 * (1 - 2 * ((e >> d) & 1)).to(torch.bfloat16)
            w[f"l{i}.mlp.router.b"] = (0.9 * ((e * 3 + 1) % E if E % 3 else e)).to(torch.bfloat16)
            w[f"l{i}.norm1"][:2] = 1
    return w


def weights(name, seed=1, steady=False):
    w = O.make_weights(CONFIGS[name], seed, RANKS[name])
    return steady_routing(CONFIGS[name], w) if steady else w


def tokens(name, n, seed=0):
    g = torch.Generator().manual_seed(100 + seed)
    return torch.randint(0, CONFIGS[name]["vocab"], (n,), generator=g).tolist()


def build_config(cfg, w, dtype, max_position=512):
    from llava_mi355x.vizosun import VizosunConfig, VizosunForCausalLM
    return VizosunForCausalLM(VizosunConfig.from_dict(cfg, {k: tuple(v.shape) for k, v in w.items()}), dtype=dtype, max_position=max_position).load_state_dict(w)


def build(name, dtype, max_position=512, w=None):
    return build_config(CONFIGS[name], w if w is not None else weights(name, steady=dtype != torch.float32), dtype, max_position)
