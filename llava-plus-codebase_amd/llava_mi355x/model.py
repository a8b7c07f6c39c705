"""Python mirror of the reference's model API over the MI355X engine (C ABI in include/llava_mi355x.h).

Same names / argument meaning / results / error behaviour as the reference classes, so `llava.serve.model_worker`,
`cli.py`, `predict.py` and the eval drivers keep working on top of it:
  LlavaConfig, LlavaLlamaModel, LlavaLlamaForCausalLM     llava/model/language_model/llava_llama.py:31-111
  LlavaMetaForCausalLM.encode_images / prepare_inputs_labels_for_multimodal   llava/model/llava_arch.py:94-240
  CLIPVisionTower (attributes callers touch)                                  llava/model/multimodal_encoder/clip_encoder.py:7-78
PyTorch tensors are containers (allocation, pointers, current stream); all arithmetic on the path runs in the HIP
kernels.  There is no CPU fallback: constructing a model without a GPU / without the built extension raises.
"""
from __future__ import annotations

import ctypes
from typing import Sequence, Dict, List, Mapping, Optional, Tuple, Union

import numpy as np
import torch

from . import _C
from ._C import LmxConfig, check, lib, ptr, stream_handle, torch_dtype_code
from .constants import IGNORE_INDEX
from .engine_lm import EngineCausalLM, LmxKVCache, _EmbedTokens

try:  # HF containers for the return type / config plumbing only
    from transformers import LlamaConfig
    from transformers.modeling_outputs import CausalLMOutputWithPast
except Exception as _e:  # pragma: no cover
    raise ImportError("transformers is required for LlamaConfig / CausalLMOutputWithPast containers") from _e


class LlavaConfig(LlamaConfig):
    """llava_llama.py:31-32.  Extra fields read by the path: mm_vision_tower, mm_hidden_size, mm_projector_type,
    mm_vision_select_layer, mm_vision_select_feature, mm_use_im_start_end, mm_use_im_patch_token, image_aspect_ratio,
    tokenizer_padding_side, tokenizer_model_max_length (llava_arch.py:48-68, train.py:935-956)."""
    model_type = "llava"


_PROJ_RE = __import__("re").compile(r"^mlp(\d+)x_gelu$")


def _projector_kind(name: str) -> Tuple[int, int]:
    if name == "linear":
        return _C.PROJ_LINEAR, 1
    if name == "identity":
        return _C.PROJ_IDENTITY, 0
    m = _PROJ_RE.match(name)
    if m:
        return _C.PROJ_MLP_GELU, int(m.group(1))
    raise ValueError(f"Unknown projector type: {name}")          # multimodal_projector/builder.py:51


class CLIPVisionTower:
    """The attributes/methods callers touch on `model.get_vision_tower()` (builder.py:139-144, model_worker.py:148):
    is_loaded, load_model(), to(), image_processor, config, hidden_size, num_patches, dtype, device, __call__."""

    def __init__(self, owner: "LlavaLlamaForCausalLM"):
        self._owner = owner
        self.is_loaded = False
        self.image_processor = None
        self.vision_tower_name = getattr(owner.config, "mm_vision_tower", None)
        self.select_layer = owner.config.mm_vision_select_layer
        self.select_feature = getattr(owner.config, "mm_vision_select_feature", "patch")

    def load_model(self):
        """clip_encoder.py:21-27: processor + weights.  Weights go straight into the engine (see builder.load_vision_tower)."""
        from .builder import load_vision_tower
        load_vision_tower(self._owner)
        self.is_loaded = True

    def to(self, *args, **kwargs):
        return self

    def requires_grad_(self, flag=False):
        return self

    @property
    def config(self):
        return self._owner.vision_config

    @property
    def hidden_size(self):
        return self._owner.vision_config.hidden_size

    @property
    def num_patches(self):
        c = self._owner.vision_config
        return (c.image_size // c.patch_size) ** 2

    @property
    def dtype(self):
        return self._owner.dtype

    @property
    def device(self):
        return self._owner.device

    @property
    def dummy_feature(self):
        return torch.zeros(1, self.hidden_size, device=self.device, dtype=self.dtype)

    def feature_rows(self) -> int:
        return self._owner.tokens_per_image

    @torch.no_grad()
    def forward(self, images):
        """clip_encoder.py:39-51: hidden_states[select_layer] (CLS dropped for 'patch'), cast back to the input dtype; a list of
        [3,S,S] images gives a list of [1,P,D] features.  (model.encode_images runs the same tower fused with the projector.)"""
        o = self._owner
        o._ensure_final()

        def run(x):
            x = x.to(device=o.device, dtype=o.dtype).contiguous()
            out = torch.empty((x.shape[0], o.tokens_per_image, self.hidden_size), dtype=o.dtype, device=o.device)
            with torch.cuda.device(o.device):
                check(lib.lmx_vision_tower(o._h, ptr(x), x.shape[0], ptr(out), stream_handle()), "lmx_vision_tower")
            return out

        if type(images) is list:
            return [run(im.unsqueeze(0)).to(im.dtype) for im in images]
        return run(images).to(images.dtype)

    __call__ = forward


class LlavaLlamaModel:
    """`model.get_model()` surface: get_vision_tower(), embed_tokens, mm_projector marker (llava_arch.py:27-40)."""

    def __init__(self, owner):
        self._owner = owner
        self.vision_tower = CLIPVisionTower(owner) if getattr(owner.config, "mm_vision_tower", None) is not None else None
        self.embed_tokens = _EmbedTokens(owner)
        self.mm_projector = getattr(owner.config, "mm_projector_type", "linear")

    def get_vision_tower(self):
        return self.vision_tower


class LlavaLlamaForCausalLM(EngineCausalLM):
    """Drop-in for llava_llama.py:40-108 on the MI355X engine."""

    config_class = LlavaConfig

    def __init__(self, config: LlavaConfig, vision_config=None, dtype: torch.dtype = torch.bfloat16, device: Union[str, torch.device] = "cuda",
                 tp_rank: int = 0, tp_world: int = 1, max_position: Optional[int] = None, gemm_variant: int = 0, vocab_headroom: int = 0):
        """vocab_headroom: spare embedding / lm_head rows so that `resize_token_embeddings(len(tokenizer))` (builder.py:138) can grow the
        vocabulary by the <im_patch> / <im_start> / <im_end> tokens after the weights were loaded; the engine tables hold
        round_up(vocab_size + headroom, 8) rows, ids >= config.vocab_size are never picked and are sliced off the logits."""
        if not torch.cuda.is_available():
            raise RuntimeError("llava_mi355x needs an MI355X (HIP) device; there is no CPU path")
        self.config = config
        self.vision_config = vision_config
        self.dtype = dtype
        self.device = torch.device(device if str(device) != "cuda" else f"cuda:{torch.cuda.current_device()}")
        self.tp_rank, self.tp_world = tp_rank, tp_world
        c = LmxConfig()
        c.abi_version = _C.LMX_ABI_VERSION
        c.dtype = torch_dtype_code(dtype)
        c.hidden_size = config.hidden_size
        c.intermediate_size = config.intermediate_size
        c.n_layers = config.num_hidden_layers
        c.n_heads = config.num_attention_heads
        c.n_kv_heads = getattr(config, "num_key_value_heads", None) or config.num_attention_heads
        c.head_dim = config.hidden_size // config.num_attention_heads
        self._vocab_cap = (int(config.vocab_size) + int(vocab_headroom) + 7) // 8 * 8
        c.vocab_size = self._vocab_cap
        c.rms_eps = config.rms_norm_eps
        c.rope_theta = float(_rope_theta(config))
        c.max_position = int(max_position or config.max_position_embeddings)
        if vision_config is not None:
            c.v_hidden = vision_config.hidden_size
            c.v_intermediate = vision_config.intermediate_size
            c.v_layers = vision_config.num_hidden_layers
            c.v_heads = vision_config.num_attention_heads
            c.v_image_size = vision_config.image_size
            c.v_patch_size = vision_config.patch_size
            c.v_ln_eps = vision_config.layer_norm_eps
            c.select_layer = config.mm_vision_select_layer
            c.select_feature = _C.FEATURE_PATCH if getattr(config, "mm_vision_select_feature", "patch") == "patch" else _C.FEATURE_CLS_PATCH
            if getattr(config, "mm_vision_select_feature", "patch") not in ("patch", "cls_patch"):
                raise ValueError(f"Unexpected select feature: {config.mm_vision_select_feature}")   # clip_encoder.py:36
            c.projector_type, c.projector_depth = _projector_kind(getattr(config, "mm_projector_type", "linear"))
        c.tp_rank, c.tp_world = tp_rank, tp_world
        c.gemm_variant = gemm_variant
        self._cfg = c
        self._h = ctypes.c_void_p()
        with torch.cuda.device(self.device):
            check(lib.lmx_create(ctypes.byref(c), ctypes.byref(self._h)), "lmx_create")
        check(lib.lmx_set_vocab_limit(self._h, int(config.vocab_size)), "lmx_set_vocab_limit")
        self.s_max = (c.max_position + 127) // 128 * 128
        self._set_rope_table()
        self.model = LlavaLlamaModel(self)
        self._init_host_state()

    @property
    def row_pitch(self) -> int:
        return self.config.hidden_size

    @property
    def logits_dtype(self) -> torch.dtype:
        return self.dtype

    def cache_geometry(self) -> Tuple[int, int, int]:
        """(layers, kv heads, head width) of a sequence's cache."""
        c = self.config
        return c.num_hidden_layers, c.num_key_value_heads, c.hidden_size // c.num_attention_heads

    @classmethod
    def from_pretrained(cls, model_path, *args, **kwargs):
        """llava/model/builder.py:100,106 call `LlavaLlamaForCausalLM.from_pretrained(path, low_cpu_mem_usage=True, config=..., **kwargs)`."""
        from .builder import from_pretrained
        return from_pretrained(model_path, *args, **kwargs)

    def _set_rope_table(self):
        """cos/sin computed on the host exactly as LlamaRotaryEmbedding does (HF5:models/llama/modeling_llama.py:73-127)."""
        D = self.config.hidden_size // self.config.num_attention_heads
        theta = _rope_theta(self.config)
        inv_freq = 1.0 / (theta ** (torch.arange(0, D, 2, dtype=torch.int64).to(torch.float32) / D))
        freqs = torch.arange(self.s_max, dtype=torch.float32)[:, None] * inv_freq[None, :]
        table = torch.cat([freqs.cos(), freqs.sin()], dim=-1).contiguous()
        check(lib.lmx_set_rope_table(self._h, ctypes.c_void_p(table.data_ptr()), self.s_max), "lmx_set_rope_table")

    # ---- weights --------------------------------------------------------------------------------------------------
    @staticmethod
    def canonical_name(key: str) -> Optional[str]:
        """Map a checkpoint key (LLaVA / HF-CLIP 4.31 / HF-CLIP 5.x layouts) to the engine's canonical name; None = skip."""
        if key.endswith("rotary_emb.inv_freq") or key.endswith("position_ids"):
            return None
        k = key
        for pre in ("model.vision_tower.vision_tower.", "vision_tower.vision_tower.", "vision_tower."):
            if k.startswith(pre):
                k = "vision::" + k[len(pre):]
                break
        if k.startswith("vision_model."):
            k = "vision::" + k
        if k.startswith("vision::"):
            k = k[len("vision::"):]
            if k.startswith("vision_model."):
                k = k[len("vision_model."):]
            if k.startswith("post_layernorm"):
                return None
            return "vision." + k
        if k.startswith("vision."):
            return None if "post_layernorm" in k else k
        if k.startswith("model.mm_projector."):
            return k[len("model."):]
        if k.startswith("embeddings.") or k.startswith("encoder.layers.") or k.startswith("pre_layrnorm."):
            return "vision." + k        # bare CLIPVisionModel keys (transformers 5.x)
        if k.startswith("post_layernorm"):
            return None
        return k

    def _shape_tensor(self, name: str, t: torch.Tensor) -> torch.Tensor:
        if name in ("model.embed_tokens.weight", "lm_head.weight") and t.shape[0] != self._vocab_cap:
            if t.shape[0] > self._vocab_cap:
                raise ValueError(f"{name} has {t.shape[0]} rows, the engine vocabulary holds {self._vocab_cap}")
            pad = torch.zeros((self._vocab_cap - t.shape[0], t.shape[1]), dtype=t.dtype, device=t.device)
            t = torch.cat([t, pad], dim=0)           # padding ids: zero rows, masked out of every pick (lmx_set_vocab_limit)
        return t

    def init_tensor_parallel(self, force_comm: bool = False, rccl: bool = True, p2p: Optional[bool] = None):
        """Create the RCCL communicator: rank 0 makes the unique id, torch.distributed (any backend) broadcasts it.
        force_comm=True builds a 1-rank communicator for an unsharded model, so every decoder all-reduce site really
        calls ncclAllReduce on the launch stream (single-GPU test of the RCCL call path).
        p2p (default: on unless LLAVA_MI355X_P2P=0): also connect the one-shot peer-to-peer all-reduce used for decode-sized
        messages; it is self-tested on every rank and switched off everywhere unless all ranks pass.
        rccl=False (tests: two ranks sharing one GPU, which RCCL refuses) skips the communicator."""
        if self.tp_world == 1 and not force_comm:
            return
        import torch.distributed as dist
        if rccl:
            buf = (ctypes.c_uint8 * 128)()
            if self.tp_rank == 0:
                check(lib.lmx_tp_unique_id(buf), "lmx_tp_unique_id")
            obj = [bytes(buf)]
            if self.tp_world > 1:
                dist.broadcast_object_list(obj, src=0)
            raw = (ctypes.c_uint8 * 128).from_buffer_copy(obj[0])
            with torch.cuda.device(self.device):
                check(lib.lmx_tp_init(self._h, raw), "lmx_tp_init")
        if p2p is None:
            import os
            p2p = os.environ.get("LLAVA_MI355X_P2P", "1") != "0"
        self.p2p_active = False
        if p2p and self.tp_world > 1:
            ok, why = True, ""
            try:
                hd = (ctypes.c_uint8 * 64)()
                with torch.cuda.device(self.device):
                    check(lib.lmx_tp_p2p_local_handle(self._h, hd), "lmx_tp_p2p_local_handle")
                mine = bytes(hd)
            except Exception as e:  # noqa: BLE001
                ok, why, mine = False, repr(e), b"\0" * 64
            # every rank takes part in the SAME sequence of host collectives whatever happens locally (a rank that skipped one
            # after a local failure would leave the others waiting in it)
            gathered = [None] * self.tp_world
            dist.all_gather_object(gathered, (ok, mine))
            if all(g[0] for g in gathered):
                try:
                    blob = b"".join(g[1] for g in gathered)
                    with torch.cuda.device(self.device):
                        check(lib.lmx_tp_p2p_connect(self._h, (ctypes.c_uint8 * len(blob)).from_buffer_copy(blob)), "lmx_tp_p2p_connect")
                except Exception as e:  # noqa: BLE001
                    ok, why = False, repr(e)
            else:
                ok = False
            connected = [None] * self.tp_world
            dist.all_gather_object(connected, ok)
            if all(connected):
                try:
                    ok, why = self._p2p_selftest()
                except Exception as e:  # noqa: BLE001
                    ok, why = False, repr(e)
            else:
                ok = False
            verdicts = [None] * self.tp_world
            dist.all_gather_object(verdicts, (ok, why))
            self.p2p_active = all(v[0] for v in verdicts)
            if not self.p2p_active:
                try:
                    lib.lmx_tp_p2p_enable(self._h, 0)
                except Exception:  # noqa: BLE001
                    pass
                if self.tp_rank == 0:
                    import warnings
                    warnings.warn(f"peer-to-peer all-reduce disabled, decode all-reduces use RCCL: {[v[1] for v in verdicts if not v[0]]}")
                if not rccl:
                    raise RuntimeError(f"p2p all-reduce self-test failed and no RCCL communicator: {verdicts}")

    def tp_comm_ranks(self) -> int:
        """Ranks in the engine's RCCL communicator (ncclCommCount); 0 when there is none."""
        return int(lib.lmx_tp_comm_ranks(self._h))

    def _p2p_selftest(self) -> Tuple[bool, str]:
        """All-reduce integer-valued rows (exact in every dtype) through the P2P kernel and compare with the closed-form sum."""
        H, W, r = self.config.hidden_size, self.tp_world, self.tp_rank
        idx = torch.arange(H, device=self.device) % 13
        for it in range(12):
            for rows in (1, 4, 32) + ((33, 577) if it < 3 else ()):                                       # > 32 rows: the two-shot (reduce-scatter + all-gather) kernel
                base = (idx[None, :] + torch.arange(rows, device=self.device)[:, None] + it) % 7          # values 0..6
                mine = (base * (r + 1)).to(self.dtype).contiguous()
                want = (base * (W * (W + 1) // 2)).to(self.dtype)
                check(lib.lmx_op_allreduce(self._h, ptr(mine), rows * H, stream_handle()), "lmx_op_allreduce")
                torch.cuda.current_stream(self.device).synchronize()
                if lib.lmx_tp_p2p_status(self._h, stream_handle()) != 0:
                    return False, f"rank {r}: wait for a peer timed out (iteration {it}, rows {rows})"
                if not torch.equal(mine, want):
                    return False, f"rank {r}: wrong sum (iteration {it}, rows {rows})"
        return True, ""

    # ---- reference API surface --------------------------------------------------------------------------------------
    def get_model(self):
        return self.model

    def get_vision_tower(self):
        return self.get_model().get_vision_tower()

    @property
    def tokens_per_image(self) -> int:
        return lib.lmx_tokens_per_image(self._h)

    def _hash_images(self, x: torch.Tensor) -> List[Tuple[int, int]]:
        """128-bit content hash per image of a contiguous [N, 3, S, S] device tensor (lmx_op_hash128); one 16 N-byte read-back."""
        n = x.shape[0]
        out = torch.empty((n, 2), dtype=torch.int64, device=self.device)
        check(lib.lmx_op_hash128(ptr(x), x[0].numel() * x.element_size(), n, ptr(out), stream_handle()), "lmx_op_hash128")
        h = out.cpu().numpy().view(np.uint64)
        # dtype and geometry are part of the key: the same bytes under another interpretation are another image
        salt = hash((str(x.dtype), tuple(x.shape[1:]))) & 0xFFFFFFFF
        return [(int(h[i, 0]) ^ salt, int(h[i, 1])) for i in range(n)]

    def _check_pixels(self, images: torch.Tensor) -> torch.Tensor:
        if self.vision_config is None:
            raise ValueError("model has no vision tower")
        x = images.to(device=self.device, dtype=self.dtype).contiguous()
        if x.dim() != 4 or x.shape[1] != 3 or x.shape[2] != self.vision_config.image_size or x.shape[3] != self.vision_config.image_size:
            raise ValueError(f"images must be [N,3,{self.vision_config.image_size},{self.vision_config.image_size}], got {tuple(x.shape)}")
        return x

    def _run_tower(self, x: torch.Tensor, out: torch.Tensor, sharded: bool) -> None:
        """Tower + projector over x [n,3,S,S] into out [n,P,H].  sharded (tensor parallel, n >= 2; a COLLECTIVE — every rank calls it with the same
        pixels at the same point of its call sequence): the tower is data parallel over the images ("split images across ranks for B > 1,
        then all-gather features") — rank r runs images r, r + W, ..., the other rows of `out` stay zero and the decoder's all-reduce sums the ranks'
        buffers, which IS the all-gather (every element has one non-zero contributor: exact in every dtype, like the vocabulary-parallel logits row)."""
        n = x.shape[0]
        if not sharded:
            check(lib.lmx_encode_images(self._h, ptr(x), n, ptr(out), stream_handle()), "lmx_encode_images")
            return
        mine = torch.arange(self.tp_rank, n, self.tp_world, device=self.device)
        out.zero_()
        if mine.numel():
            xm = x.index_select(0, mine).contiguous()
            om = torch.empty((int(mine.numel()),) + tuple(out.shape[1:]), dtype=out.dtype, device=out.device)
            check(lib.lmx_encode_images(self._h, ptr(xm), int(mine.numel()), ptr(om), stream_handle()), "lmx_encode_images")
            out.index_copy_(0, mine, om)
        # pieces of <= 4096 rows of H elements: what the two-shot peer-to-peer all-reduce takes in one launch (engine.cpp: p2p_big_max_count)
        per = max(1, 4096 // max(1, out.shape[1] * out.shape[2] // self.config.hidden_size))
        for i0 in range(0, n, per):
            piece = out[i0:i0 + per]
            check(lib.lmx_op_allreduce(self._h, ptr(piece), piece.numel(), stream_handle()), "lmx_op_allreduce")

    def tower_is_sharded(self, n_images: int) -> bool:
        """Whether encode_images_sharded() would split n_images over the tensor-parallel ranks (LLAVA_MI355X_TP_TOWER=0 keeps the tower replicated)."""
        import os
        return self.tp_world > 1 and n_images >= 2 and os.environ.get("LLAVA_MI355X_TP_TOWER", "1") != "0"

    def encode_images_sharded(self, images: torch.Tensor) -> torch.Tensor:
        """encode_images for the images of a whole BATCH of requests under tensor parallelism: the ranks split the images and all-gather the features
        (_run_tower).  COLLECTIVE: every rank must call it with the same pixels, in step with its other engine calls — generate_batch and
        tp_serving.prefill_symmetric do; a request thread's own encode_images never is (the tower stays replicated there)."""
        return self.encode_images(images, _collective=True)

    def encode_images(self, images: torch.Tensor, _collective: bool = False) -> torch.Tensor:
        """llava_arch.py:94-97 — images [N,3,S,S] -> [N, tokens_per_image, hidden].  With enable_reuse(): images whose pixels were encoded before return
        the stored rows (reuse.ImageFeatureCache), only the others run the tower."""
        ov = getattr(self._tls, "feats_override", None)
        if ov is not None:
            # features of this request's images were computed with the batch's (generate_batch / prefill_symmetric: encode_images_sharded)
            self._tls.feats_override = None
            feats, hashes = ov
            if feats.shape[0] != images.shape[0]:
                raise ValueError(f"pre-encoded features cover {feats.shape[0]} images, the request has {images.shape[0]}")
            self._tls.image_hashes = hashes
            return feats
        x = self._check_pixels(images)
        self._ensure_final()
        n = x.shape[0]
        P = self.tokens_per_image
        out = torch.empty((n, P, self.config.hidden_size), dtype=self.dtype, device=self.device)
        cache = self._img_cache
        self._tls.image_hashes = None
        if cache is None or n == 0:
            self._run_tower(x, out, _collective and self.tower_is_sharded(n))
            return out
        hashes = self._hash_images(x)
        self._tls.image_hashes = hashes
        stored = [cache.get(h) for h in hashes]
        miss = [i for i in range(n) if stored[i] is None]
        if miss:
            # the caches of all ranks hold the same entries (same calls in the same order), so the miss list — and with it the split — is the same everywhere
            sharded = _collective and self.tower_is_sharded(len(miss))
            if len(miss) == n:
                self._run_tower(x, out, sharded)
                fresh = out
            else:
                xm = x.index_select(0, torch.tensor(miss, device=self.device)).contiguous()
                fresh = torch.empty((len(miss), P, self.config.hidden_size), dtype=self.dtype, device=self.device)
                self._run_tower(xm, fresh, sharded)
            for j, i in enumerate(miss):
                if fresh is not out:
                    out[i].copy_(fresh[j])
                cache.put(hashes[i], fresh[j].clone())
        for i in range(n):
            if stored[i] is not None:
                out[i].copy_(stored[i])
        return out

    def _preencode_local(self, images_per_request: Sequence):
        """Rank-local half of the sharded tower pass over the images of several requests (tensor parallel): geometry checks, the concatenation, the output
        buffer and THIS rank's share of the images through the tower — everything that can fail on one rank alone (a device copy, an allocation), and
        nothing collective.  The split is a function of the image count only (rank r takes images r, r + W, ...; the image-feature cache is NOT consulted
        here: a cache that diverged between ranks must not change who encodes what).  Returns None when there is nothing to shard, else the state for
        _preencode_collective.  images_per_request: per request a [k,3,S,S] tensor, None, or anything else (left to the request's own, replicated, encode)."""
        idx = [i for i, im in enumerate(images_per_request) if isinstance(im, torch.Tensor) and im.dim() == 4 and im.shape[0] > 0]
        if not idx or not self.tower_is_sharded(sum(int(images_per_request[i].shape[0]) for i in idx)):
            return None
        self._ensure_final()
        cat = torch.cat([self._check_pixels(images_per_request[i]) for i in idx], dim=0)
        n = int(cat.shape[0])
        out = torch.zeros((n, self.tokens_per_image, self.config.hidden_size), dtype=self.dtype, device=self.device)
        mine = torch.arange(self.tp_rank, n, self.tp_world, device=self.device)
        if mine.numel():
            xm = cat.index_select(0, mine).contiguous()
            om = torch.empty((int(mine.numel()),) + tuple(out.shape[1:]), dtype=out.dtype, device=out.device)
            check(lib.lmx_encode_images(self._h, ptr(xm), int(mine.numel()), ptr(om), stream_handle()), "lmx_encode_images")
            out.index_copy_(0, mine, om)
        return {"idx": idx, "counts": [int(images_per_request[i].shape[0]) for i in idx], "n_req": len(images_per_request), "cat": cat, "out": out}

    def _preencode_collective(self, st) -> List:
        """COLLECTIVE half: the ranks' buffers are summed (every element has one non-zero contributor: the sum IS the all-gather, exact in every dtype).
        Only launches all-reduces on buffers that already exist.  Returns per request None or the (features [k,P,H], image hashes) pair that
        `_tls.feats_override` hands to the request's encode_images; with enable_reuse() the features also enter the image-feature cache."""
        out = st["out"]
        n = int(out.shape[0])
        # pieces of <= 4096 rows of H elements: what the two-shot peer-to-peer all-reduce takes in one launch (engine.cpp: p2p_big_max_count)
        per = max(1, 4096 // max(1, out.shape[1] * out.shape[2] // self.config.hidden_size))
        for i0 in range(0, n, per):
            piece = out[i0:i0 + per]
            check(lib.lmx_op_allreduce(self._h, ptr(piece), piece.numel(), stream_handle()), "lmx_op_allreduce")
        hashes = None
        if self._img_cache is not None:
            hashes = self._hash_images(st["cat"])
            for i, h in enumerate(hashes):
                if self._img_cache.get(h) is None:
                    self._img_cache.put(h, out[i].clone())
        res: List = [None] * st["n_req"]
        o = 0
        for i, k in zip(st["idx"], st["counts"]):
            res[i] = (out[o:o + k], None if hashes is None else hashes[o:o + k])
            o += k
        return res

    def _preencode_requests(self, images_per_request: Sequence) -> List:
        """The images of several requests through ONE sharded tower pass (tensor parallel; a COLLECTIVE): rank-local half + collective half back to back,
        for callers whose ranks run in lock step by construction (generate_batch).  The serving path brackets the halves with agreements
        (tp_serving.prefill_symmetric)."""
        st = self._preencode_local(images_per_request)
        return [None] * len(images_per_request) if st is None else self._preencode_collective(st)

    def prepare_inputs_labels_for_multimodal(self, input_ids, position_ids, attention_mask, past_key_values, labels, images):
        """llava_arch.py:99-240, same 6-tuple.  Integer half on the host through lmx_splice_plan (bit-exact), embedding
        gather/splice on the device."""
        vision_tower = self.get_vision_tower()
        if vision_tower is None or images is None or input_ids.shape[1] == 1:
            if past_key_values is not None and vision_tower is not None and images is not None and input_ids.shape[1] == 1:
                target_shape = past_key_values[-1][-1].shape[-2] + 1                  # llava_arch.py:105
                attention_mask = torch.cat((attention_mask, torch.ones((attention_mask.shape[0], target_shape - attention_mask.shape[1]),
                                                                       dtype=attention_mask.dtype, device=attention_mask.device)), dim=1)
                position_ids = torch.sum(attention_mask, dim=1).unsqueeze(-1) - 1
            return input_ids, position_ids, attention_mask, past_key_values, None, labels

        if type(images) is list or images.ndim == 5:                                   # llava_arch.py:114-119
            concat = torch.cat([im for im in images], dim=0)
            feats = self.encode_images(concat)
            P = feats.shape[1]
            slot_rows = np.asarray([im.shape[0] * P for im in images], dtype=np.int32)
            feat_mat = feats.reshape(-1, feats.shape[-1])
        else:
            feats = self.encode_images(images)
            P = feats.shape[1]
            slot_rows = None
            feat_mat = feats.reshape(-1, feats.shape[-1])
        n_slots = len(images) if slot_rows is not None else feats.shape[0]

        if getattr(self.config, "tune_mm_mlp_adapter", False) and getattr(self.config, "mm_use_im_start_end", False):
            raise NotImplementedError                                                   # llava_arch.py:124-125

        ids_h = np.ascontiguousarray(input_ids.detach().cpu().numpy().astype(np.int64))        # same D2H the reference does (:161)
        B, L = ids_h.shape
        mask_h = None if attention_mask is None else np.ascontiguousarray(attention_mask.detach().cpu().numpy().astype(np.uint8))
        lab_h = None if labels is None else np.ascontiguousarray(labels.detach().cpu().numpy().astype(np.int64))
        max_len = getattr(self.config, "tokenizer_model_max_length", None) or 0
        left = getattr(self.config, "tokenizer_padding_side", "right") == "left"
        vp = lambda a: ctypes.c_void_p(0) if a is None else ctypes.c_void_p(a.ctypes.data)
        T = ctypes.c_int32(0)
        args = (vp(ids_h), vp(mask_h), vp(lab_h), B, L, P, vp(slot_rows), n_slots, int(max_len), int(left))
        rc = lib.lmx_splice_plan(*args, ctypes.byref(T), None, None, None, None)
        if rc:
            raise IndexError(_C.last_error())          # the reference raises IndexError on image_features[cur_image_idx]
        Tn = T.value
        src = np.empty((B, Tn), np.int32); om = np.empty((B, Tn), np.uint8)
        op = np.empty((B, Tn), np.int64); ol = np.empty((B, Tn), np.int64)
        check(lib.lmx_splice_plan(*args, ctypes.byref(T), vp(src), vp(om), vp(op), vp(ol)), "lmx_splice_plan")
        if (src >= self.config.vocab_size).any():
            raise IndexError("token id out of range for embed_tokens")
        src_d = torch.from_numpy(src).to(self.device)
        embeds = torch.empty((B, Tn, self.config.hidden_size), dtype=self.dtype, device=self.device)
        check(lib.lmx_gather_embeds(self._h, ptr(src_d), B * Tn, ptr(feat_mat.to(self.dtype).contiguous()), ptr(embeds), stream_handle()), "lmx_gather_embeds")
        dev = input_ids.device
        new_labels = None if labels is None else torch.from_numpy(ol).to(device=labels.device, dtype=labels.dtype)
        new_mask = None if attention_mask is None else torch.from_numpy(om).to(device=attention_mask.device, dtype=attention_mask.dtype)
        new_pos = None if position_ids is None else torch.from_numpy(op).to(device=position_ids.device, dtype=position_ids.dtype)
        # keep the plan's mask for the decoder even when the caller passed attention_mask=None
        self._tls.plan_mask = torch.from_numpy(om.astype(bool))
        self._tls.plan_src, self._tls.plan_P = src, P           # row identities for the prefix cache (reuse.row_keys)
        return None, new_pos, new_mask, past_key_values, embeds, new_labels

    # ---- decoder ---------------------------------------------------------------------------------------------------
    def _prefill_rows_outputs(self, cache: LmxKVCache, embeds: torch.Tensor, valid: Optional[torch.Tensor], want_hidden: bool, want_attn: bool):
        """_prefill_rows(want_all=True) that also returns `output_hidden_states`' tuple — L + 1 tensors [B,T,H]: entry l < L = the rows entering decoder layer l,
        entry L = the final norm's output (HF5:models/llama/modeling_llama.py:367-418) — and / or `output_attentions`' tuple — L tensors [B, heads, T, past + T]:
        each layer's post-softmax attention weights as the eager path returns them (:191-214), recomputed from the rotated q rows and the K cache
        (lmx_prefill_outputs).  Pad rows / pad key columns stay zero."""
        B, T, H = embeds.shape
        V, L, nh = self._vocab_cap, self.config.num_hidden_layers, self.config.num_attention_heads
        past = cache.lengths()
        logits = torch.zeros((B, T, V), dtype=self.dtype, device=self.device)
        hidden = torch.zeros((L + 1, B, T, H), dtype=self.dtype, device=self.device) if want_hidden else None
        attn = None
        if want_attn:
            if self.tp_world > 1:
                raise NotImplementedError("output_attentions under tensor parallelism: every rank holds a slice of the heads")
            if any(p > 0 for p in past) and valid is not None and not bool(valid.all()):
                raise NotImplementedError("output_attentions with padding on top of a KV cache is not supported (un-padded continuation, or padded batches from an empty cache)")
            attn = torch.zeros((L, B, nh, T, max(past) + T), dtype=self.dtype, device=self.device)
        for b in range(B):
            idx = None
            if valid is not None:
                idx = torch.nonzero(valid[b].to(self.device), as_tuple=False).flatten()
                if int(idx.numel()) == T:
                    idx = None
                elif int(idx.numel()) == 0:
                    continue
            e = (embeds[b] if idx is None else embeds[b].index_select(0, idx)).contiguous()
            n = e.shape[0]
            lg = torch.empty((n, V), dtype=self.dtype, device=self.device)
            hs = torch.empty((L + 1, n, H), dtype=self.dtype, device=self.device) if want_hidden else None
            ap = torch.empty((L, nh, n, past[b] + n), dtype=self.dtype, device=self.device) if want_attn else None
            check(lib.lmx_prefill_outputs(self._h, cache.seqs[b], ptr(e), n, ptr(lg), 1, ptr(hs), ptr(ap), stream_handle()), "lmx_prefill_outputs")
            if idx is None:
                logits[b] = lg
                if want_hidden:
                    hidden[:, b] = hs
                if want_attn:
                    attn[:, b, :, :, : past[b] + n] = ap
            else:
                logits[b].index_copy_(0, idx, lg)
                if want_hidden:
                    hidden[:, b].index_copy_(1, idx, hs)
                if want_attn:
                    attn[:, b][:, :, idx[:, None], idx[None, :]] = ap           # past == 0 here: compacted rows / keys back to their padded places
        return (logits, None if hidden is None else tuple(hidden[l] for l in range(L + 1)), None if attn is None else tuple(attn[l] for l in range(L)))

    def forward(self, input_ids=None, attention_mask=None, position_ids=None, past_key_values=None, inputs_embeds=None, labels=None,
                use_cache=None, output_attentions=None, output_hidden_states=None, images=None, return_dict=None, **kwargs):
        """llava_llama.py:56-99.  Returns CausalLMOutputWithPast(loss, logits [B,T,V] fp32 (as transformers 4.31 does),
        past_key_values=LmxKVCache).  Pad positions (attention_mask == 0) get zero logits.  output_hidden_states=True (llava_llama.py:63-64)
        adds `hidden_states`, LlamaModel's tuple of L + 1 tensors [B,T,H] (pad rows zero); output_attentions=True (llava_llama.py:62-63) adds `attentions`, the
        tuple of L tensors [B, heads, T, past + T] the eager attention returns (pad rows / columns zero) — recomputed beside the fused kernels for this call only."""
        hidden_states, attentions = None, None
        want_out = bool(output_hidden_states) or bool(output_attentions)
        self._ensure_final()
        user_pos = position_ids
        plan_mask = None
        if inputs_embeds is None:
            self._tls.plan_mask = None
            (input_ids, position_ids, attention_mask, past_key_values, inputs_embeds, labels) = self.prepare_inputs_labels_for_multimodal(
                input_ids, position_ids, attention_mask, past_key_values, labels, images)
            plan_mask = self._tls.plan_mask
        if inputs_embeds is None:
            inputs_embeds = self.get_model().embed_tokens(input_ids)
        inputs_embeds = inputs_embeds.to(device=self.device, dtype=self.dtype)
        B, T, _ = inputs_embeds.shape
        if past_key_values is not None and not isinstance(past_key_values, LmxKVCache):
            raise TypeError("past_key_values must come from this model (LmxKVCache)")
        decode_step = past_key_values is not None and T == 1 and input_ids is not None
        if decode_step:
            cache = past_key_values
            V = self._vocab_cap
            logits = torch.empty((B, 1, V), dtype=self.dtype, device=self.device)
            toks = input_ids.reshape(-1).tolist()
            if position_ids is not None:
                want = torch.tensor(cache.lengths(), dtype=torch.long)
                if not torch.equal(position_ids.reshape(-1).cpu().long(), want):
                    raise ValueError("position_ids must continue each sequence's cache (the fused RoPE derives positions from the KV-cache length)")
            if want_out:
                # one position through the prefill path, which can hand out the layer inputs / attention rows (the decode kernels keep them in their workspace only)
                logits, hidden_states, attentions = self._prefill_rows_outputs(cache, inputs_embeds, None, bool(output_hidden_states), bool(output_attentions))
            else:
                for b in range(B):
                    check(lib.lmx_decode(self._h, cache.seqs[b], int(toks[b]), 1, ptr(logits[b]), 0, stream_handle()), "lmx_decode")
        else:
            cache = past_key_values if past_key_values is not None else LmxKVCache(self, B)
            valid = None
            if attention_mask is not None:
                valid = attention_mask[:, -T:].bool()
            elif plan_mask is not None:
                valid = plan_mask
            # position_ids are implied by the mask (consecutive over each row's unmasked tokens, exactly what the splice
            # builds at llava_arch.py:206-223 and what HF derives when none are given); anything else is refused, not ignored.
            if position_ids is not None:
                base = torch.tensor(cache.lengths(), dtype=torch.long)[:, None]
                ok = torch.ones((B, T), dtype=torch.bool) if valid is None else valid.cpu().bool()
                want = (torch.cumsum(ok.long(), dim=1) - 1).clamp_min(0) + base
                got = position_ids[:, -T:].cpu().long().expand(B, T)
                if not torch.equal(got[ok], want[ok]):
                    raise ValueError("non-consecutive position_ids are not supported: the fused RoPE numbers each row's unmasked tokens 0, 1, 2, ...")
            if want_out:
                logits, hidden_states, attentions = self._prefill_rows_outputs(cache, inputs_embeds, valid, bool(output_hidden_states), bool(output_attentions))
            else:
                logits = self._prefill_rows(cache, inputs_embeds, valid, want_all=True, greedy=False)
        logits = logits[..., : self.config.vocab_size].float()        # padded ids (engine row pitch) are not part of the vocabulary
        loss = None
        if labels is not None:
            # LlamaForCausalLM's shifted cross-entropy (logits[..., :-1, :] vs labels[..., 1:], IGNORE_INDEX skipped, mean) on the
            # device: csrc/train.hip ce_fwd_kernel, fp32 math on the fp32 logits exactly as transformers 4.31 upcasts them
            from . import ops
            lab = labels.to(device=logits.device, dtype=torch.long).contiguous()
            loss, _, _ = ops.ce_loss(logits.contiguous(), lab, ignore_index=IGNORE_INDEX)
        if use_cache is False and past_key_values is None:
            cache.close()
            cache = None
        if return_dict is False:
            return tuple(x for x in (loss, logits, cache, hidden_states, attentions) if x is not None)
        return CausalLMOutputWithPast(loss=loss, logits=logits, past_key_values=cache, hidden_states=hidden_states, attentions=attentions)

    __call__ = forward

    def prepare_inputs_for_generation(self, input_ids, past_key_values=None, inputs_embeds=None, **kwargs):
        """llava_llama.py:101-108: HF's default slicing + re-attached `images`."""
        images = kwargs.pop("images", None)
        if past_key_values is not None:
            input_ids = input_ids[:, -1:]
        out = {"input_ids": input_ids, "past_key_values": past_key_values, "use_cache": kwargs.get("use_cache"),
               "attention_mask": kwargs.get("attention_mask")}
        if inputs_embeds is not None and past_key_values is None:
            out = {"inputs_embeds": inputs_embeds, **{k: v for k, v in out.items() if k != "input_ids"}}
        if images is not None:
            out["images"] = images
        return out


def _rope_theta(config) -> float:
    t = getattr(config, "rope_theta", None)
    if t is None:
        rp = getattr(config, "rope_parameters", None) or {}
        t = rp.get("rope_theta", 10000.0) if isinstance(rp, dict) else 10000.0
    return float(t)
