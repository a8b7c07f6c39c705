"""Configurations and helpers of the Siterax tests: small, unequal sizes on purpose (no two numbers of a layer are equal unless the case is about that)."""
import json
import os

import torch

from oracle import siterax_oracle as O


def layer(heads, kv, dim, vdim, window, rot_dims, ff, base=10000.0, factor=1.0, scale=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5,
                                           "mask": {"size": window} if window else None, "rot": {"dims": rot_dims, "base": base, "scaling": {"factor": factor}}},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(layers, width, vocab, loop=None, mult=0.7, cap=20.0, eps=1e-5):
    return {"architecture": "Siterax", "layers": layers, "width": width, "vocab": vocab, "loop": loop, "residual_mult": mult, "logit_softcap": cap, "norm": {"eps": eps}}


CONFIGS = {
    # every layer another shape, a layer without feed-forward, the loop in the middle, partial rotation with and without whole 16-element groups
    "mixed": config([layer(4, 2, 48, 64, 24, 32, 160, base=5000.0, factor=3.0), layer(6, 1, 64, 32, 0, 64, 0), layer(3, 3, 80, 80, 130, 20, 96, factor=1.5),
                     layer(2, 1, 36, 52, 7, 6, 224)], 192, 203, {"start": 1, "stop": 3, "times": 3}),
    # sizes off every padding boundary, a window of one key, no loop
    "odd": config([layer(5, 1, 72, 40, 1, 72, 50), layer(2, 2, 20, 12, 65, 4, 33)], 100, 97, None, mult=1.0, cap=30.0, eps=1e-3),
    # head vectors wider than 128
    "wide": config([layer(2, 1, 160, 200, 40, 96, 128, factor=4.0)], 128, 64, {"start": 0, "stop": 1, "times": 2}),
    # one head, equal sizes, one pass, everything looped; width a whole 512
    "single": config([layer(1, 1, 128, 128, 128, 128, 512, scale=0.2)] * 2, 512, 512, {"start": 0, "stop": 2, "times": 1}, mult=0.25, cap=8.0),
}


def weights(name, seed=1):
    return O.make_weights(CONFIGS[name], seed)


def tokens(name, n, seed=0):
    g = torch.Generator().manual_seed(100 + seed)
    return torch.randint(0, CONFIGS[name]["vocab"], (n,), generator=g).tolist()


def save_checkpoint(path, cfg, w):
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in w.items()}, os.path.join(path, "model.safetensors"))


def build(name, dtype, max_position=512, w=None):
    from llava_mi355x.siterax import SiteraxConfig, SiteraxForCausalLM
    m = SiteraxForCausalLM(SiteraxConfig.from_dict(CONFIGS[name]), dtype=dtype, max_position=max_position)
    return m.load_state_dict(w if w is not None else weights(name))


def rel(got, want):
    """Root mean square of the difference over that of the reference, worst row."""
    got, want = got.detach().double().cpu(), want.double()
    return ((got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()).max().item()
