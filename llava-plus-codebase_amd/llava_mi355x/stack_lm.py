"""What the layer-stack families (siterax.py, vizosun.py) share on the host: an engine handle described layer by layer (lmx_create_stack), loading, prefill with chosen
logits and forward().  A family supplies its configuration class and the two engine descriptions made from it."""
from __future__ import annotations

import ctypes
from dataclasses import dataclass
from typing import Optional, Sequence, Tuple

import torch

from . import _C
from ._C import LmxLayerConfig, LmxStackConfig, check, lib, ptr, stream_handle, torch_dtype_code
from .engine_lm import EngineCausalLM, LmxKVCache, _EmbedTokens


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


class StackCausalLM(EngineCausalLM):
    config_class: type

    def describe(self, c: LmxStackConfig, layers: Sequence[LmxLayerConfig]) -> None:
        """Fill the engine's description from self.config (abi_version, dtype, sizes common to all families and max_position are set)."""
        raise NotImplementedError

    def create_tables(self) -> None:
        """Host-made tables the engine needs before its first use."""

    def __init__(self, config, dtype: torch.dtype = torch.bfloat16, device="cuda", max_position: Optional[int] = None, gemm_variant: int = 0):
        if not torch.cuda.is_available():
            raise RuntimeError("llava_mi355x needs an MI355X (HIP) device; there is no CPU path")
        self.config, self.dtype = config, dtype
        self.device = torch.device(device if str(device) != "cuda" else f"cuda:{torch.cuda.current_device()}")
        c = LmxStackConfig()
        c.abi_version, c.dtype = _C.LMX_ABI_VERSION, torch_dtype_code(dtype)
        c.width, c.vocab_size, c.n_layers = config.width, config.vocab_size, len(config.layers)
        c.max_position = int(max_position or config.max_position)
        c.loop_start, c.loop_stop, c.loop_times = config.loop
        c.norm_eps, c.residual_mult = config.norm_eps, 1.0
        c.gemm_variant = gemm_variant
        arr = (LmxLayerConfig * len(config.layers))()
        self.describe(c, arr)
        self._h = ctypes.c_void_p()
        with torch.cuda.device(self.device):
            check(lib.lmx_create_stack(ctypes.byref(c), arr, ctypes.byref(self._h)), "lmx_create_stack")
        self.s_max = (c.max_position + 127) // 128 * 128
        self.create_tables()
        self.row_pitch = lib.lmx_input_pitch(self._h)
        self._vocab_cap = lib.lmx_vocab_pitch(self._h)
        self.logits_dtype = torch.float32
        self.exact_prefixes = lib.lmx_recurrent(self._h) == 1
        self.model = _TextModel(self)
        self._init_host_state()

    @classmethod
    def from_pretrained(cls, path: str, torch_dtype: Optional[torch.dtype] = None, device="cuda", max_position: Optional[int] = None, **_unused) -> "StackCausalLM":
        from .registry import iter_checkpoint
        model = cls(cls.config_class.from_pretrained(path), dtype=torch_dtype or torch.bfloat16, device=device, max_position=max_position)
        for k, v in iter_checkpoint(path):
            model.load_tensor(k, v)
        model.finalize_weights()
        return model

    def cache_geometry(self) -> Tuple[int, int, int]:
        """(cache slots, kv heads, head width): what `past_key_values` shows of its shape; a latent row or a recurrent state counts as one head."""
        mixers = [getattr(x, "mixer", x) for x in self.config.layers]
        return lib.lmx_layer_runs(self._h), max(getattr(m, "kv_heads", 1) for m in mixers), max(m.dim for m in mixers)

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
                hidden = torch.empty((B, runs, T, lib.lmx_row_pitch(self._h)), dtype=torch.float32, device=self.device)
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
