"""Siterax: a small decoder-only language model with normed sublayers on both sides, per-head query / key norms, sliding windows with a softmax sink, per-head output
gates and a range of layers that runs several times.  Host side only: configuration, tensor names and rotary tables; the layers run on the engine's layer-stack decoder
(csrc/stack.cpp) through the same sequences, batches, scheduler and samplers as every other model of the package."""
from __future__ import annotations

import ctypes
import json
import os
from dataclasses import dataclass, field
from typing import Any, Dict, List, Mapping, Optional, Tuple

import torch

from . import _C
from ._C import LmxLayerConfig, LmxStackConfig, check, lib, ptr, stream_handle, torch_dtype_code
from .engine_lm import EngineCausalLM, LmxKVCache, _EmbedTokens


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


@dataclass
class CausalLMOutput:
    logits: torch.Tensor
    past_key_values: Optional[LmxKVCache] = None
    hidden_states: Optional[torch.Tensor] = None      # [layer runs, B, T, width] fp32: the residual stream after every layer run


class _TextModel:
    """`get_model()` of a text-only family."""

    def __init__(self, owner: EngineCausalLM):
        self.embed_tokens = _EmbedTokens(owner)

    def get_vision_tower(self):
        return None


def rotary_table(rot: RotaryConfig, n_pos: int) -> torch.Tensor:
    """[n_pos, dims] fp32: cosines of the pairs' angles, then sines.  Angles in float64: an fp32 angle is off by up to 2^-24 of the position."""
    half = rot.dims // 2
    freq = rot.base ** (-2.0 * torch.arange(half, dtype=torch.float64) / rot.dims) / rot.factor
    ang = torch.arange(n_pos, dtype=torch.float64)[:, None] * freq[None, :]
    return torch.cat([ang.cos(), ang.sin()], dim=1).to(torch.float32).contiguous()


class SiteraxForCausalLM(EngineCausalLM):
    config_class = SiteraxConfig

    def __init__(self, config: SiteraxConfig, dtype: torch.dtype = torch.bfloat16, device="cuda", max_position: Optional[int] = None, gemm_variant: int = 0):
        if not torch.cuda.is_available():
            raise RuntimeError("llava_mi355x needs an MI355X (HIP) device; there is no CPU path")
        self.config, self.dtype = config, dtype
        self.device = torch.device(device if str(device) != "cuda" else f"cuda:{torch.cuda.current_device()}")
        c = LmxStackConfig()
        c.abi_version, c.dtype = _C.LMX_ABI_VERSION, torch_dtype_code(dtype)
        c.width, c.vocab_size, c.n_layers = config.width, config.vocab_size, len(config.layers)
        c.max_position = int(max_position or config.max_position)
        c.loop_start, c.loop_stop, c.loop_times = config.loop
        c.norm_eps, c.residual_mult, c.logit_softcap = config.norm_eps, config.residual_mult, config.logit_softcap
        c.gemm_variant = gemm_variant
        rots: List[RotaryConfig] = []
        arr = (LmxLayerConfig * len(config.layers))()
        for a, l in zip(arr, config.layers):
            a.n_heads, a.n_kv_heads, a.qk_dim, a.v_dim = l.heads, l.kv_heads, l.dim, l.vdim
            a.attn_scale, a.window, a.softmax_sink, a.qk_norm, a.qkv_bias, a.out_gate = l.scale, l.window, 1, 1, 1, 1
            a.rope_dims, a.ff = l.rot.dims, l.ff
            if l.rot.dims:
                if l.rot not in rots:
                    rots.append(l.rot)
                a.rope_table = rots.index(l.rot)
        self._h = ctypes.c_void_p()
        with torch.cuda.device(self.device):
            check(lib.lmx_create_stack(ctypes.byref(c), arr, ctypes.byref(self._h)), "lmx_create_stack")
        self.s_max = (c.max_position + 127) // 128 * 128
        for i, r in enumerate(rots):
            table = rotary_table(r, self.s_max)
            check(lib.lmx_stack_set_rope(self._h, i, r.dims, ctypes.c_void_p(table.data_ptr()), self.s_max), "lmx_stack_set_rope")
        self.row_pitch = lib.lmx_row_pitch(self._h)
        self._vocab_cap = lib.lmx_vocab_pitch(self._h)
        self.logits_dtype = torch.float32
        self.model = _TextModel(self)
        self._init_host_state()

    @classmethod
    def from_pretrained(cls, path: str, torch_dtype: Optional[torch.dtype] = None, device="cuda", max_position: Optional[int] = None, **_unused) -> "SiteraxForCausalLM":
        from .registry import iter_checkpoint
        model = cls(SiteraxConfig.from_pretrained(path), dtype=torch_dtype or torch.bfloat16, device=device, max_position=max_position)
        for k, v in iter_checkpoint(path):
            model.load_tensor(k, v)
        model.finalize_weights()
        return model

    def cache_geometry(self) -> Tuple[int, int, int]:
        l = self.config.layers
        return lib.lmx_layer_runs(self._h), max(x.kv_heads for x in l), max(x.dim for x in l)

    def prefill_logits(self, caches, embeds, wants) -> torch.Tensor:
        n, total = len(caches), sum(len(w) for w in wants)
        logits = torch.empty((total, self._vocab_cap), dtype=torch.float32, device=self.device)
        embeds = [e.to(self.dtype).contiguous() for e in embeds]
        arr = (ctypes.c_void_p * n)(*[c.seqs[0].value for c in caches])
        eptr = (ctypes.c_void_p * n)(*[e.data_ptr() for e in embeds])
        cnt = (ctypes.c_int32 * n)(*[e.shape[0] for e in embeds])
        nw = (ctypes.c_int32 * n)(*[len(w) for w in wants])
        wr = (ctypes.c_int32 * max(1, total))(*[int(r) for w in wants for r in w])
        check(lib.lmx_prefill_batch_logits(self._h, arr, n, eptr, cnt, 0, nw, wr, ptr(logits), 0, stream_handle()), "lmx_prefill_batch_logits")
        return logits

    @torch.inference_mode()
    def forward(self, input_ids: torch.Tensor, past_key_values: Optional[LmxKVCache] = None, use_cache: bool = True, output_hidden_states: bool = False, chunk: int = 0,
                **_unused) -> CausalLMOutput:
        """Logits [B, T, vocab] fp32 of un-padded rows, continuing past_key_values when given.  A single new token per row goes through the decode kernels."""
        self._ensure_final()
        B, T = input_ids.shape
        cache = past_key_values if past_key_values is not None else LmxKVCache(self, B)
        V, hidden = self._vocab_cap, None
        if past_key_values is not None and T == 1 and not output_hidden_states:
            logits = torch.empty((B, 1, V), dtype=torch.float32, device=self.device)
            for b, t in enumerate(input_ids.reshape(-1).tolist()):
                check(lib.lmx_decode(self._h, cache.seqs[b], int(t), 1, ptr(logits[b]), 0, stream_handle()), "lmx_decode")
        else:
            embeds = self.get_model().embed_tokens(input_ids)
            if output_hidden_states:
                runs = lib.lmx_layer_runs(self._h)
                logits = torch.empty((B, T, V), dtype=torch.float32, device=self.device)
                hidden = torch.empty((B, runs, T, self.row_pitch), dtype=torch.float32, device=self.device)
                for b in range(B):
                    check(lib.lmx_prefill_hidden(self._h, cache.seqs[b], ptr(embeds[b]), T, ptr(logits[b]), 1, ptr(hidden[b]), stream_handle()), "lmx_prefill_hidden")
                hidden = hidden[..., : self.config.width].transpose(0, 1)
            else:
                logits = self._prefill_rows(cache, embeds, None, want_all=True, greedy=False, chunk=chunk)
        if not use_cache and past_key_values is None:
            torch.cuda.current_stream(self.device).synchronize()
            cache.close()
            cache = None
        return CausalLMOutput(logits[..., : self.config.vocab_size], cache, hidden)

    __call__ = forward
