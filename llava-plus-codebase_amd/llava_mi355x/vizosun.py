"""Vizosun: a small decoder-only language model whose layers run mixer and feed-forward side by side on one norm.  Mixers are latent attention (low-rank queries, keys and
values, no positions, sliding window) and a gated delta rule with a decay per key channel; feed-forwards are dense (ReLU-gated) or mixtures of experts (SiLU-gated); a
bigram table joins the token embedding; a range of layers may run several times, each pass beginning with a projection of the stream and the embedding output.  Host side
only: configuration and tensor names; the layers run on the engine's layer-stack decoder (csrc/stack.cpp, csrc/stack_mixers.cpp)."""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field
from typing import Any, Dict, List, Mapping, Optional, Sequence, Tuple

from . import _C
from ._C import LmxLayerConfig, LmxStackConfig
from .stack_lm import StackCausalLM


@dataclass(frozen=True)
class LatentMixer:
    heads: int
    dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    window: int                      # 0: every earlier position


@dataclass(frozen=True)
class DeltaMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int
    decay_rank: int                  # inner sizes of the decay and output-gate projections: known from their tensors only
    gate_rank: int


@dataclass(frozen=True)
class VizosunLayer:
    mixer: Any                       # LatentMixer | DeltaMixer
    ff: int                          # 0: no feed-forward; of one expert where there are experts
    experts: int = 0
    top: int = 0


@dataclass(frozen=True)
class BigramConfig:
    buckets: int
    mul_prev: int
    mul_cur: int


@dataclass
class VizosunConfig:
    vocab_size: int
    width: int
    layers: List[VizosunLayer]
    norm_eps: float
    bigram: Optional[BigramConfig] = None
    loop: Tuple[int, int, int] = (0, 0, 1)      # start, stop, times
    looped: bool = False
    max_position: int = 4096
    eos_token_id: Optional[int] = None
    pad_token_id: Optional[int] = None
    extra: Dict[str, Any] = field(default_factory=dict)

    @classmethod
    def from_dict(cls, d: Mapping[str, Any], shapes: Mapping[str, Sequence[int]]) -> "VizosunConfig":
        """`shapes`: tensor shapes of the checkpoint (registry.checkpoint_shapes), for the sizes the configuration does not name."""
        layers = []
        for i, e in enumerate(d["layers"]):
            m, mlp = e["mixer"], e.get("mlp")
            if e["type"] == "latent_attention":
                mixer = LatentMixer(int(m["heads"]), int(m["dim"]), int(m["vdim"]), int(m["q_rank"]), int(m["kv_rank"]), float(m["scale"]), int((m.get("mask") or {}).get("size") or 0))
            elif e["type"] == "channel_delta":
                mixer = DeltaMixer(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), int(m["conv"]), int(shapes[f"l{i}.mix.a1"][0]), int(shapes[f"l{i}.mix.g1"][0]))
            else:
                raise ValueError(f"layer {i}: unknown mixer type {e['type']!r}")
            if mlp is None:
                layers.append(VizosunLayer(mixer, 0))
            elif mlp["kind"] == "dense":
                layers.append(VizosunLayer(mixer, int(mlp["ff"])))
            elif mlp["kind"] == "moe":
                layers.append(VizosunLayer(mixer, int(mlp["expert"]["ff"]), int(mlp["router"]["experts"]), int(mlp["router"]["top"])))
            else:
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
        lp, bg = d.get("loop"), (d.get("embedding") or {}).get("bigram")
        known = ("architecture", "embedding", "layers", "loop", "norm", "vocab", "width", "max_position", "eos_token_id", "pad_token_id")
        return cls(vocab_size=int(d["vocab"]), width=int(d["width"]), layers=layers, norm_eps=float(d["norm"]["eps"]),
                   bigram=None if not bg else BigramConfig(int(bg["buckets"]), int(bg["mul_prev"]), int(bg["mul_cur"])),
                   loop=(0, 0, 1) if not lp else (int(lp["start"]), int(lp["stop"]), int(lp["times"])), looped=bool(lp),
                   max_position=int(d.get("max_position") or 4096), eos_token_id=d.get("eos_token_id"), pad_token_id=d.get("pad_token_id"),
                   extra={k: v for k, v in d.items() if k not in known})

    @classmethod
    def from_pretrained(cls, path: str) -> "VizosunConfig":
        from .registry import checkpoint_shapes
        with open(os.path.join(path, "config.json")) as f:
            return cls.from_dict(json.load(f), checkpoint_shapes(path))

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)


class VizosunForCausalLM(StackCausalLM):
    config_class = VizosunConfig

    def describe(self, c: LmxStackConfig, layers: Sequence[LmxLayerConfig]) -> None:
        g = self.config
        c.tied_head, c.loop_mix = 1, int(g.looped)
        if g.bigram is not None:
            c.bigram_buckets, c.bigram_mul_prev, c.bigram_mul_cur = g.bigram.buckets, g.bigram.mul_prev, g.bigram.mul_cur
        for a, l in zip(layers, g.layers):
            m = l.mixer
            a.n_heads, a.n_kv_heads, a.qk_dim, a.v_dim, a.parallel = m.heads, m.heads, m.dim, m.vdim, 1
            if isinstance(m, LatentMixer):
                a.mixer, a.q_rank, a.kv_rank, a.attn_scale, a.window = _C.MIXER_LATENT, m.q_rank, m.kv_rank, m.scale, m.window
            else:
                a.mixer, a.n_kv_heads, a.conv_taps, a.decay_rank, a.gate_rank = _C.MIXER_DELTA, m.kv_heads, m.taps, m.decay_rank, m.gate_rank
            a.ff, a.experts, a.top_experts = l.ff, l.experts, l.top
            a.ff_act = _C.ACT_SILU_MUL if l.experts else _C.ACT_RELU_MUL
