"""Siterax: a small decoder-only language model with normed sublayers on both sides, per-head query / key norms, sliding windows with a softmax sink, per-head output
gates and a range of layers that runs several times.  Host side only: configuration, tensor names and rotary tables; the layers run on the engine's layer-stack decoder
(csrc/stack.cpp) through the same sequences, batches, scheduler and samplers as every other model of the package."""
from __future__ import annotations

import ctypes
import json
import os
from dataclasses import dataclass, field
from typing import Any, Dict, List, Mapping, Optional, Sequence, Tuple

import torch

from ._C import LmxLayerConfig, LmxStackConfig, check, lib
from .stack_lm import CausalLMOutput, StackCausalLM  # noqa: F401


@dataclass(frozen=True)
class RotaryConfig:
    dims: int = 0                    # leading dimensions rotated (0: none)
    base: float = 10000.0
    factor: float = 1.0              # linear scaling: every frequency is divided by it


@dataclass(frozen=True)
class SiteraxLayer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int                      # 0: every earlier position
    rot: RotaryConfig
    ff: int                          # 0: no feed-forward


@dataclass
class SiteraxConfig:
    vocab_size: int
    width: int
    layers: List[SiteraxLayer]
    norm_eps: float
    residual_mult: float = 1.0
    logit_softcap: float = 0.0       # 0: none
    loop: Tuple[int, int, int] = (0, 0, 1)      # start, stop, times
    max_position: int = 4096
    eos_token_id: Optional[int] = None
    pad_token_id: Optional[int] = None
    extra: Dict[str, Any] = field(default_factory=dict)

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "SiteraxConfig":
        layers = []
        for i, e in enumerate(d["layers"]):
            if e["type"] != "attention":
                raise ValueError(f"layer {i}: unknown mixer type {e['type']!r}")
            m, mlp = e["mixer"], e.get("mlp")
            if mlp is not None and mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
            rot = m.get("rot")
            rotary = RotaryConfig() if rot is None else RotaryConfig(int(rot["dims"]), float(rot["base"]), float((rot.get("scaling") or {}).get("factor", 1.0)))
            layers.append(SiteraxLayer(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), float(m["scale"]), int((m.get("mask") or {}).get("size") or 0),
                                       rotary, 0 if mlp is None else int(mlp["ff"])))
        lp = d.get("loop")
        known = ("architecture", "layers", "loop", "norm", "vocab", "width", "residual_mult", "logit_softcap", "max_position", "eos_token_id", "pad_token_id")
        return cls(vocab_size=int(d["vocab"]), width=int(d["width"]), layers=layers, norm_eps=float(d["norm"]["eps"]), residual_mult=float(d.get("residual_mult", 1.0)),
                   logit_softcap=float(d.get("logit_softcap") or 0.0), loop=(0, 0, 1) if not lp else (int(lp["start"]), int(lp["stop"]), int(lp["times"])),
                   max_position=int(d.get("max_position") or 4096), eos_token_id=d.get("eos_token_id"), pad_token_id=d.get("pad_token_id"),
                   extra={k: v for k, v in d.items() if k not in known})

    @classmethod
    def from_pretrained(cls, path: str) -> "SiteraxConfig":
        with open(os.path.join(path, "config.json")) as f:
            return cls.from_dict(json.load(f))

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)


def rotary_table(rot: RotaryConfig, n_pos: int) -> torch.Tensor:
    """[n_pos, dims] fp32: cosines of the pairs' angles, then sines.  Angles in float64: an fp32 angle is off by up to 2^-24 of the position."""
    half = rot.dims // 2
    freq = rot.base ** (-2.0 * torch.arange(half, dtype=torch.float64) / rot.dims) / rot.factor
    ang = torch.arange(n_pos, dtype=torch.float64)[:, None] * freq[None, :]
    return torch.cat([ang.cos(), ang.sin()], dim=1).to(torch.float32).contiguous()


class SiteraxForCausalLM(StackCausalLM):
    config_class = SiteraxConfig

    def describe(self, c: LmxStackConfig, layers: Sequence[LmxLayerConfig]) -> None:
        c.residual_mult, c.logit_softcap = self.config.residual_mult, self.config.logit_softcap
        self._rots: List[RotaryConfig] = []
        for a, l in zip(layers, self.config.layers):
            a.n_heads, a.n_kv_heads, a.qk_dim, a.v_dim = l.heads, l.kv_heads, l.dim, l.vdim
            a.attn_scale, a.window, a.softmax_sink, a.qk_norm, a.qkv_bias, a.out_gate = l.scale, l.window, 1, 1, 1, 1
            a.rope_dims, a.ff = l.rot.dims, l.ff
            if l.rot.dims:
                if l.rot not in self._rots:
                    self._rots.append(l.rot)
                a.rope_table = self._rots.index(l.rot)

    def create_tables(self) -> None:
        for i, r in enumerate(self._rots):
            table = rotary_table(r, self.s_max)
            check(lib.lmx_stack_set_rope(self._h, i, r.dims, ctypes.c_void_p(table.data_ptr()), self.s_max), "lmx_stack_set_rope")
