"""Host side of the engine shared by every causal language model of this package: lifetime and weights of an engine handle, sequences, packed prefill, offline batches,
generate() (greedy, sampled, beams, streaming, stop rules), the continuous-batching scheduler and the prefix cache.

A model family is a subclass: it creates the engine handle (`_h`) from its own configuration and may add inputs of its own (model.py: images spliced into the prompt).
What a subclass has to provide: config (vocab_size, optional eos / pad ids), dtype, logits_dtype, device, s_max, row_pitch (elements of an embedding row), _vocab_cap (elements
of a logits row), tp_rank / tp_world, cache_geometry() and get_model().embed_tokens.
PyTorch tensors are containers (allocation, pointers, current stream); all arithmetic on the path runs in the HIP kernels."""
from __future__ import annotations

import ctypes
import threading
from typing import Dict, List, Mapping, Optional, Sequence, Tuple

import numpy as np
import torch

from ._C import check, lib, ptr, stream_handle, torch_dtype_code
from .constants import IMAGE_TOKEN_INDEX


class LmxKVCache:
    """`past_key_values` of this build: one engine sequence (KV cache + device decode state) per batch row.
    Supports the one access the reference makes — `past_key_values[-1][-1].shape[-2]` (llava_arch.py:105)."""

    class _Shape:
        def __init__(self, shape):
            self.shape = shape

    def __init__(self, model: "EngineCausalLM", batch: int):
        self.model = model
        self.seqs: List[ctypes.c_void_p] = []
        for _ in range(batch):
            h = ctypes.c_void_p()
            check(lib.lmx_seq_create(model._h, ctypes.byref(h)), "lmx_seq_create")
            self.seqs.append(h)

    def lengths(self) -> List[int]:
        return [lib.lmx_seq_length(s) for s in self.seqs]

    def get_seq_length(self, layer_idx: int = 0) -> int:
        return max(self.lengths()) if self.seqs else 0

    def __len__(self):
        return self.model.cache_geometry()[0]

    def __getitem__(self, i):
        _, kv_heads, head_dim = self.model.cache_geometry()
        shp = (len(self.seqs), kv_heads, self.get_seq_length(), head_dim)
        return (self._Shape(shp), self._Shape(shp))

    def close(self):
        for s in self.seqs:
            lib.lmx_seq_destroy(s)
        self.seqs = []

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass


class _EmbedTokens:
    def __init__(self, owner):
        self._owner = owner

    def __call__(self, ids: torch.Tensor) -> torch.Tensor:
        o = self._owner
        flat = ids.reshape(-1).to(device=o.device, dtype=torch.int32).contiguous()
        if flat.numel() and bool(((flat < 0) | (flat >= o.config.vocab_size)).any()):
            raise IndexError("index out of range in self")          # what nn.Embedding raises for an id beyond the (resized) vocabulary
        out = torch.empty((flat.numel(), o.row_pitch), dtype=o.dtype, device=o.device)
        if flat.numel():
            check(lib.lmx_gather_embeds(o._h, ptr(flat), flat.numel(), None, ptr(out), stream_handle()), "gather_embeds")
        return out.view(*ids.shape, o.row_pitch)


class EngineCausalLM:
    """A causal language model on one engine handle; see the module docstring for what a subclass provides."""

    tp_rank, tp_world = 0, 1
    exact_prefixes = False              # sequences carry state that cannot be cut back (lmx_recurrent): a prefix is reused whole or not at all

    def _init_host_state(self) -> None:
        self.generation_config = None
        self._lock = threading.Lock()
        self._tls = threading.local()       # per-request scratch (model_worker runs several generate threads on one model)
        self._batcher = None                # continuous-batching scheduler (enable_batching)
        self._prefill_gate = threading.Semaphore(1)
        self._batch_prefill_chunk = 0
        self._finalized = False
        self._img_cache = None              # reuse.ImageFeatureCache / reuse.PrefixCache (enable_reuse): off by default
        self._prefix = None

    # ---- what a family with more than token ids as input overrides ------------------------------------------------------
    @staticmethod
    def canonical_name(key: str) -> Optional[str]:
        """Engine name of a checkpoint key; None = not loaded."""
        return key

    def _shape_tensor(self, name: str, t: torch.Tensor) -> torch.Tensor:
        return t

    def get_model(self):
        return self.model

    def get_vision_tower(self):
        return None

    def prepare_inputs_labels_for_multimodal(self, input_ids, position_ids, attention_mask, past_key_values, labels, images):
        if images is not None:
            raise ValueError("this model takes token ids only")
        return input_ids, position_ids, attention_mask, past_key_values, None, labels

    def _preencode_requests(self, images_per_request: Sequence) -> List:
        return [None] * len(images_per_request)

    def __del__(self):
        try:
            if getattr(self, "_h", None):
                lib.lmx_destroy(self._h)
                self._h = None
        except Exception:
            pass

    def load_tensor(self, name: str, tensor: torch.Tensor) -> None:
        t = tensor.detach().to(device=self.device, dtype=self.dtype).contiguous()
        t = self._shape_tensor(name, t).contiguous()
        self._finalized = False
        shape = (ctypes.c_int64 * t.dim())(*t.shape)
        check(lib.lmx_load_weight(self._h, name.encode(), ptr(t), torch_dtype_code(self.dtype), t.dim(), shape, stream_handle()),
              f"lmx_load_weight({name})")
        torch.cuda.current_stream().synchronize()      # `t` may be a temporary; the copy must land before it is freed

    def load_state_dict(self, state: Mapping[str, torch.Tensor], strict: bool = True):
        for k, v in state.items():
            name = self.canonical_name(k)
            if name is None:
                continue
            self.load_tensor(name, v)
        if strict:
            self.finalize_weights()
        return self

    def finalize_weights(self):
        check(lib.lmx_finalize_weights(self._h), "lmx_finalize_weights")
        self._finalized = True

    def _ensure_final(self):
        """The reference has no explicit 'weights complete' step (from_pretrained + vision_tower.load_model()); the engine's
        completeness check therefore runs on first use."""
        if not self._finalized:
            self.finalize_weights()

    def set_option(self, key: str, value: int) -> None:
        """Flip one of the engine's launch-form options ("fuse_rope", "vis_pack", "decode_splitq": bit-identical forms; include/llava_mi355x.h)."""
        check(lib.lmx_model_set_option(self._h, key.encode(), int(value)), "lmx_model_set_option")

    def profile(self, enable: bool) -> None:
        check(lib.lmx_profile_enable(self._h, int(enable)), "lmx_profile_enable")

    def profile_read(self) -> Dict[str, Tuple[float, int]]:
        """{launch-group name: (total ms, launches)} accumulated since profile(True)."""
        names = ctypes.create_string_buffer(16384)
        ms = (ctypes.c_double * 256)(); cnt = (ctypes.c_int64 * 256)(); n = ctypes.c_int32(0)
        check(lib.lmx_profile_read(self._h, names, 16384, ms, cnt, 256, ctypes.byref(n)), "lmx_profile_read")
        keys = names.value.decode().split("\n")[: n.value]
        return {k: (ms[i], cnt[i]) for i, k in enumerate(keys)}

    def eval(self):
        return self

    def to(self, *args, **kwargs):
        return self

    def half(self):
        return self

    def cuda(self, *a, **k):
        return self

    def requires_grad_(self, flag=False):
        return self

    def resize_token_embeddings(self, n: int):
        """builder.py:138 calls this after adding <im_patch> / <im_start> / <im_end>.  The engine tables were allocated with headroom
        (`vocab_headroom`), so growing or shrinking the REAL vocabulary inside that capacity is a limit change: new ids get zero
        embedding / lm_head rows (the reference leaves them untrained too), ids >= n are never picked and are sliced off the logits."""
        n = int(n)
        if n < 1 or n > self._vocab_cap:
            raise ValueError(f"resize_token_embeddings({n}): the engine vocabulary holds {self._vocab_cap} rows; construct the model "
                             f"with vocab_headroom >= {n - int(self.config.vocab_size)}")
        check(lib.lmx_set_vocab_limit(self._h, n), "lmx_set_vocab_limit")
        self.config.vocab_size = n
        return self.get_model().embed_tokens

    def enable_reuse(self, images: int = 64, prefixes: int = 32, min_rows: int = 32) -> None:
        """Switch on the two caches of reuse.py: image features by pixel content (`images` entries of tokens_per_image x hidden each) and KV prefixes of
        finished requests (`prefixes` sequences: ~0.5 MB per position at 7B).  Off by default; bench.py never enables them.  Prefix reuse is a single-process
        feature (tensor-parallel followers replay the leader's calls; their caches would have to make the same decisions — not wired)."""
        from .reuse import ImageFeatureCache, PrefixCache
        self.disable_reuse()
        if images > 0:
            self._img_cache = ImageFeatureCache(images)
        if prefixes > 0 and self.tp_world == 1:
            self._prefix = PrefixCache(prefixes, min_rows)

    def disable_reuse(self) -> None:
        if self._prefix is not None:
            self._prefix.clear()
        self._img_cache, self._prefix = None, None

    def reuse_stats(self) -> dict:
        ic, pc = self._img_cache, self._prefix
        return {"image_hits": ic.hits if ic else 0, "image_misses": ic.misses if ic else 0, "prefix_hits": pc.hits if pc else 0,
                "prefix_misses": pc.misses if pc else 0, "prefix_rows_reused": pc.rows_reused if pc else 0, "prefix_entries": len(pc) if pc else 0}

    def clear_image_cache(self) -> None:
        """Drop every stored image feature (after a failure that may have left the tensor-parallel ranks' caches different)."""
        if self._img_cache is not None:
            self._img_cache.clear()

    def prefill_logits(self, caches: Sequence["LmxKVCache"], embeds: Sequence[torch.Tensor], wants: Sequence[Sequence[int]]) -> torch.Tensor:
        """Continue several one-sequence caches by the rows in `embeds` ([T_i, row_pitch]) and return the logits of chosen rows, [sum len(wants[i]), _vocab_cap], in order
        (`wants[i]`: ascending row indices of portion i).  A family whose engine serves that in one packed prefill overrides this."""
        rows = []
        for c, e, w in zip(caches, embeds, wants):
            lg = self._prefill_rows(c, e[None], None, want_all=True, greedy=False)[0]
            rows.append(lg[list(w)])
        return torch.cat(rows)

    def _prefill_rows(self, cache: LmxKVCache, embeds: torch.Tensor, valid: Optional[torch.Tensor], want_all: bool, greedy: bool, chunk: int = 0):
        """Run the decoder over [B,T,H] embeddings; `valid` [B,T] bool marks real (non-pad) positions."""
        B, T, H = embeds.shape
        V = self._vocab_cap                 # row pitch of the engine's logits; callers slice to config.vocab_size
        logits = torch.zeros((B, T if want_all else 1, V), dtype=self.logits_dtype, device=self.device)
        for b in range(B):
            if valid is not None:
                idx = torch.nonzero(valid[b].to(self.device), as_tuple=False).flatten()
                n = int(idx.numel())
                if n == 0:
                    continue
                e = embeds[b] if n == T else embeds[b].index_select(0, idx).contiguous()
            else:
                idx, n, e = None, T, embeds[b]
            e = e.contiguous()
            if want_all:
                lg = logits[b] if n == T else torch.empty((n, V), dtype=self.logits_dtype, device=self.device)
                check(lib.lmx_prefill(self._h, cache.seqs[b], ptr(e), n, chunk, ptr(lg), 1, int(greedy), stream_handle()), "lmx_prefill")
                if n != T:
                    logits[b].index_copy_(0, idx, lg)
            else:
                check(lib.lmx_prefill(self._h, cache.seqs[b], ptr(e), n, chunk, ptr(logits[b]), 0, int(greedy), stream_handle()), "lmx_prefill")
        return logits

    def enable_batching(self, capacity: int = 32, prefill_chunk: int = 0, prewarm: bool = True, channel=None, packed_prefill: bool = True,
                        max_prefill_batch: int = 8, max_prefill_rows: int = 2304, prefill_thread: int = 2) -> None:
        """From now on concurrent generate() calls (model_worker.py:174-185 runs one thread per request) decode together:
        one scheduler thread steps every live request through lmx_decode_batch.  packed_prefill (default): the scheduler also prefills — the requests
        waiting at that moment (up to max_prefill_batch) go through lmx_prefill_batch together, between two decode steps; packed_prefill=False keeps
        each prefill on its request's own thread and stream (one at a time), where the running decode batch interleaves with it at kernel
        granularity.  `max_prefill_rows` bounds the rows of one packed prefill (default 2304: two single-image 512-token requests), i.e. how long the live requests
        wait between two of their decode steps (~18 ms per 1k rows at 7B) and the packed workspace; 0 = up to max_prefill_batch requests whatever
        their size (best burst throughput, unbounded stall).  `prefill_chunk` > 0 bounds the rows per prefill piece (workspace; costs GEMM efficiency).
        prefill_thread (single process only) = 2 (default): the packed prefills run on their own thread and stream beside the decode steps instead
        of between two of them — a new request does not wait behind the step in flight, the live requests do not wait for its prefill — and each request's
        rank-local half (image encode / feature-cache hit, splice, prefix-cache take) runs on the request's own thread before it queues; 1 = that half on the
        prefill thread too; 0 = round 4's order (one loop: prefill, then step)."""
        from .batching import DecodeBatcher
        if self.tp_world > 1:
            # tensor parallel: only the leader schedules, and it needs the command channel to its followers (tp_serving.py)
            if self.tp_rank != 0:
                raise RuntimeError("tensor-parallel rank > 0 does not schedule: run tp_serving.serve_follower(model, channel)")
            if channel is None:
                raise RuntimeError("enable_batching under tensor parallelism needs channel=tp_serving.CommandChannel(group)")
        if self._batcher is None:
            self._ensure_final()
            self._batcher = DecodeBatcher(self, capacity, channel=channel if self.tp_world > 1 else None, scheduler_prefill=bool(packed_prefill),
                                          max_prefill_batch=int(max_prefill_batch), max_prefill_rows=int(max_prefill_rows), prefill_thread=int(prefill_thread))
            self._batch_prefill_chunk = int(prefill_chunk)
            if prewarm:
                # allocate (and zero) the KV caches of `capacity` sequences now; closing them parks them in the engine's sequence
                # pool, so the first burst of requests does not pay hipMalloc + a 1 GB memset each in front of its prefill
                warm = [LmxKVCache(self, 1) for _ in range(int(capacity))]
                for c in warm:
                    c.close()

    def disable_batching(self) -> None:
        if self._batcher is not None:
            self._batcher.close()
            self._batcher = None

    @torch.no_grad()
    def generate_batch(self, prompts, images=None, max_new_tokens: int = 20, eos_token_id=None, run_ahead: int = 16,
                       prefill_chunk: int = 0, capacity: Optional[int] = None, attention_masks=None, do_sample: bool = False,
                       temperature: float = 1.0, top_p: Optional[float] = None, top_k: Optional[int] = None, packed_prefill: bool = True):
        """Offline batch generation (greedy, or sampled on the device): the requests are prefilled TOGETHER (own image, own prompt length — no padding: their
        rows form one packed block walked in pieces of prefill_chunk x requests rows, every linear a single GEMM per piece; lmx_prefill_batch), then
        all of them decode together, `run_ahead` chained steps per host round trip; finished requests leave the batch.  packed_prefill=False prefills
        request by request (lmx_prefill, `prefill_chunk` rows at a time).
        prompts: list of LongTensor [L_i] / [1, L_i] (with -200 markers); images: list of per-request tensors or None.
        Returns a list of LongTensor [L_i + new_i] (input ids echoed, like generate())."""
        from .batching import DecodeBatch
        self._ensure_final()
        n_req = len(prompts)
        images = images if images is not None else [None] * n_req
        eos = eos_token_id if eos_token_id is not None else getattr(self.config, "eos_token_id", None)
        eos_set = set(eos if isinstance(eos, (list, tuple)) else ([eos] if eos is not None else []))
        caches, outs, budgets, packed = [], [], [], []
        batch = DecodeBatch(self, capacity or max(1, n_req))
        try:
            greedy = (not do_sample) or (temperature is not None and temperature <= 1e-5)
            masks = attention_masks if attention_masks is not None else [None] * n_req
            # tensor parallel: the images of ALL requests through one tower pass split over the ranks (every rank runs this same plan)
            pre = self._preencode_requests(images) if self.tp_world > 1 else [None] * n_req
            for ids, img, am, ov in zip(prompts, images, masks, pre):
                ids = ids if ids.dim() == 2 else ids[None]
                am = None if am is None else (am if am.dim() == 2 else am[None])
                self._tls.plan_mask = None
                self._tls.feats_override = ov
                try:
                    _, _, mask, _, embeds, _ = self.prepare_inputs_labels_for_multimodal(ids, None, am, None, None, img)
                finally:
                    self._tls.feats_override = None
                if embeds is None:
                    embeds = self.get_model().embed_tokens(ids.to(self.device)); valid = None if am is None else am.bool()
                else:
                    valid = self._tls.plan_mask if mask is None else mask.bool()
                cache = LmxKVCache(self, 1)
                caches.append(cache)
                self._set_stop(cache.seqs[0], self._stop_spec(eos_set))     # a member that reached EOS stops advancing inside the batched steps
                if not greedy:
                    seed = self._draw_seed()
                    check(lib.lmx_seq_set_sampling(cache.seqs[0], float(temperature), float(top_p if top_p is not None else 1.0), int(top_k or 0), seed),
                          "lmx_seq_set_sampling")
                if packed_prefill:
                    # rows of this request for the packed prefill: its valid (non-pad) positions, in order
                    e = embeds[0]
                    if valid is not None and not bool(valid[0].all()):
                        e = e.index_select(0, torch.nonzero(valid[0].to(self.device), as_tuple=False).flatten())
                    packed.append(e.to(self.dtype).contiguous())
                else:
                    self._prefill_rows(cache, embeds, valid, want_all=False, greedy=True, chunk=prefill_chunk)
            if packed_prefill:
                n = len(packed)
                arr = (ctypes.c_void_p * n)(*[c.seqs[0].value if isinstance(c.seqs[0], ctypes.c_void_p) else c.seqs[0] for c in caches])
                eptr = (ctypes.c_void_p * n)(*[e.data_ptr() for e in packed])
                cnt = (ctypes.c_int32 * n)(*[int(e.shape[0]) for e in packed])
                check(lib.lmx_prefill_batch(self._h, arr, n, eptr, cnt, int(prefill_chunk) * n if prefill_chunk else 0, 1, stream_handle()), "lmx_prefill_batch")
            for cache in caches:
                budgets.append(min(max_new_tokens, self.s_max - lib.lmx_seq_length(cache.seqs[0])))
                host1 = (ctypes.c_int64 * 1)(); n1 = ctypes.c_int32(0)
                check(lib.lmx_seq_read_tokens(cache.seqs[0], host1, 1, ctypes.byref(n1), stream_handle()), "read_tokens")
                outs.append([int(host1[0])] if budgets[-1] > 0 else [])
            live = [i for i in range(n_req) if budgets[i] > 1 and not (outs[i] and outs[i][-1] in eos_set)]
            while live:
                for g0 in range(0, len(live), batch.capacity):
                    grp = live[g0:g0 + batch.capacity]
                    k = max(1, min([run_ahead] + [budgets[i] - len(outs[i]) for i in grp]))
                    ids_steps = batch.step([caches[i].seqs[0] for i in grp], None, k, True)
                    for j, i in enumerate(grp):
                        for st in range(k):
                            if len(outs[i]) >= budgets[i] or (outs[i] and outs[i][-1] in eos_set) or ids_steps[st][j] < 0:
                                break
                            outs[i].append(ids_steps[st][j])
                live = [i for i in live if len(outs[i]) < budgets[i] and outs[i][-1] not in eos_set]
            res = []
            for ids, o in zip(prompts, outs):
                flat = ids.reshape(-1).cpu()
                res.append(torch.cat([flat, torch.tensor(o, dtype=torch.long)]).to(self.device))
            return res
        finally:
            batch.close()
            for c in caches:
                c.close()

    @torch.inference_mode()
    def generate(self, inputs=None, images=None, do_sample=False, temperature=1.0, top_p=None, top_k=None, num_beams=1,
                 max_new_tokens=None, max_length=None, streamer=None, stopping_criteria=None, use_cache=True, attention_mask=None,
                 eos_token_id=None, pad_token_id=None, input_ids=None, run_ahead: int = 16, prefill_chunk: int = 0, **kwargs):
        """Greedy / temperature+top-p generation with the device-resident decode loop (model_worker.py:174-185 contract:
        returns LongTensor [B, L + new] that echoes the input ids, image markers included)."""
        if inputs is None:
            inputs = input_ids
        if inputs is None:
            raise ValueError("generate() needs `inputs` (input_ids)")
        self._ensure_final()
        if not use_cache:
            raise NotImplementedError("generate() always uses the KV cache")
        ids = inputs if inputs.dim() == 2 else inputs[None]
        B, L = ids.shape
        if max_new_tokens is None:
            max_new_tokens = (max_length - L) if max_length is not None else 20
        eos = eos_token_id if eos_token_id is not None else getattr(self.config, "eos_token_id", None)
        eos_set = set(eos if isinstance(eos, (list, tuple)) else ([eos] if eos is not None else []))
        pad = pad_token_id if pad_token_id is not None else (getattr(self.config, "pad_token_id", None) or 0)
        greedy = (not do_sample) or (temperature is not None and temperature <= 1e-5)
        rows: List[List[int]] = []
        if num_beams != 1:
            # GenerationMixin.beam_search / beam_sample + BeamSearchScorer (llava_mi355x/beam.py); transformers refuses a streamer here as well
            if streamer is not None:
                raise ValueError("`streamer` cannot be used with beam search (as in transformers)")
            from .beam import beam_search
            beam_images = self._row_images(ids, images, attention_mask)      # row b's own images (llava_arch.py:150-159 slot arithmetic)
            for b in range(B):
                row_mask = None if attention_mask is None else attention_mask[b:b + 1]
                rows.append(beam_search(self, ids[b:b + 1], beam_images[b], row_mask, int(num_beams), int(max_new_tokens), eos_set, float(kwargs.get("length_penalty", 1.0)),
                                        kwargs.get("early_stopping", False), prefill_chunk, bool(kwargs.get("length_counts_prompt", True)),
                                        eos_first=(eos[0] if isinstance(eos, (list, tuple)) and eos else (eos if isinstance(eos, int) and eos >= 0 else None)),
                                        stopping_criteria=list(stopping_criteria) if stopping_criteria else None,
                                        # num_beams > 1 with do_sample=True: GenerationMixin.beam_sample (beam.py)
                                        sample=None if greedy else dict(temperature=float(temperature), top_p=top_p, top_k=top_k, seed=self._draw_seed())))
            width = L + max(len(r) for r in rows)
            out = torch.full((B, width), pad, dtype=torch.long)
            for b, r in enumerate(rows):
                out[b, :L] = ids[b].cpu()
                out[b, L:L + len(r)] = torch.tensor(r, dtype=torch.long)
            return out.to(ids.device)
        if streamer is not None:
            if B != 1:
                raise ValueError("streaming needs batch size 1")
            streamer.put(ids.cpu())
        row_images = self._row_images(ids, images, attention_mask)
        if B > 1 and streamer is None and not stopping_criteria and max_new_tokens > 0:
            # rows decode together (one pass over the weights per step for the whole batch)
            outs = self.generate_batch([ids[b] for b in range(B)], row_images, max_new_tokens=max_new_tokens, eos_token_id=list(eos_set) or -1,
                                       run_ahead=run_ahead, prefill_chunk=prefill_chunk,
                                       attention_masks=None if attention_mask is None else [attention_mask[b] for b in range(B)],
                                       do_sample=not greedy, temperature=temperature, top_p=top_p, top_k=top_k)
            rows = [o[L:].tolist() for o in outs]
        else:
            for b in range(B):
                row_mask = None if attention_mask is None else attention_mask[b:b + 1]
                rows.append(self._generate_one(ids[b:b + 1], row_images[b], row_mask, greedy, temperature, top_p, top_k, max_new_tokens,
                                               eos_set, streamer, stopping_criteria, run_ahead, prefill_chunk))
        if streamer is not None:
            streamer.end()
        if self.tp_world > 1 and getattr(self, "p2p_active", False):
            st = lib.lmx_tp_p2p_status(self._h, stream_handle())
            if st != 0:
                raise RuntimeError(f"tensor-parallel rank {self.tp_rank}: peer-to-peer all-reduce #{st} timed out waiting for a peer")
        width = L + max(len(r) for r in rows)
        out = torch.full((B, width), pad, dtype=torch.long)
        for b, r in enumerate(rows):
            out[b, :L] = ids[b].cpu()
            out[b, L:L + len(r)] = torch.tensor(r, dtype=torch.long)
        return out.to(ids.device)

    @staticmethod
    def _row_images(ids, images, attention_mask) -> List:
        """A batch shares one `images` argument: row b owns the next max(1, #markers) entries, the slot arithmetic of llava_arch.py:150-159 (a text-only
        row still consumes one slot)."""
        B = ids.shape[0]
        if images is None or B == 1:
            return [images] * B
        row_images, nxt = [], 0
        for b in range(B):
            valid_ids = ids[b] if attention_mask is None else ids[b][attention_mask[b].bool().to(ids.device)]
            n_img = max(1, int((valid_ids == IMAGE_TOKEN_INDEX).sum().item()))
            row_images.append(images[nxt:nxt + n_img]); nxt += n_img
        return row_images

    def _draw_seed(self) -> int:
        """Seed of a request's device sampler, from torch's CPU generator (torch.manual_seed makes a request reproducible).  Under
        tensor parallelism every rank must draw the SAME token from the same logits — ranks that diverge feed different ids into the
        shared all-reduces — so rank 0's seed is broadcast (one more call in the identical host-collective sequence of the ranks)."""
        seed = int(torch.randint(0, 2 ** 62, (1,)).item())
        if self.tp_world > 1:
            import torch.distributed as dist
            if not (dist.is_available() and dist.is_initialized()):
                raise RuntimeError("sampled generation under tensor parallelism needs torch.distributed (rank 0's sampler seed is broadcast)")
            box = [seed]
            dist.broadcast_object_list(box, src=0)
            seed = int(box[0])
        return seed

    @staticmethod
    def _stop_spec(eos_set, criteria=None):
        """The id rules of a request's stop test in the form lmx_seq_set_stop takes them: (eos ids, keyword id lists) or None.  EOS ids: `eos_token_id` of
        generate(); keyword ids: `keyword_ids` of every KeywordsStoppingCriteria-like object among the stopping criteria (llava/mm_utils.py:83-100 builds
        them from the worker's "stop" string).  Rules the device cannot hold (more than 4 ids / keywords, a keyword longer than 8 ids) are left to the
        host alone — which evaluates every criterion on the ids it reads back in any case; the device rule only keeps ids past the stop from being made."""
        eos = sorted(int(e) for e in eos_set if e is not None and int(e) >= 0)
        kws: List[List[int]] = []
        for c in (criteria or []):
            for k in (getattr(c, "keyword_ids", None) or []):
                ids = [int(v) for v in (k.tolist() if hasattr(k, "tolist") else list(k))]
                if ids:
                    kws.append(ids)
        if len(eos) > 4:
            eos = []
        if len(kws) > 4 or any(len(k) > 8 for k in kws):
            kws = []
        return (eos, kws) if (eos or kws) else None

    def _set_stop(self, seq, spec) -> None:
        if not spec:
            return
        eos, kws = spec
        e = (ctypes.c_int64 * max(1, len(eos)))(*eos)
        flat = [v for k in kws for v in k]
        f = (ctypes.c_int64 * max(1, len(flat)))(*flat)
        ln = (ctypes.c_int32 * max(1, len(kws)))(*[len(k) for k in kws])
        check(lib.lmx_seq_set_stop(seq, e, len(eos), f, ln, len(kws), stream_handle()), "lmx_seq_set_stop")

    def _prepare_request(self, ids, images, attention_mask, sampling, stop=None, feats=None) -> dict:
        """The RANK-LOCAL half of a request's prefill: image encode (the tower is replicated here; `feats` = the (features, hashes) pair of a batch-wide
        sharded pass, _preencode_requests, replaces it), splice, selection of the valid rows, a fresh sequence with its
        sampling state.  Nothing in here carries a decoder collective, so under tensor parallelism a failure (a bad request, an allocation) can still be
        agreed on by all ranks before the collective-bearing half runs (tp_serving.prefill_symmetric).  Returns {cache, embeds, valid}."""
        cache = None
        try:
            self._tls.plan_mask = None
            self._tls.plan_src = None
            self._tls.feats_override = feats
            try:
                _, _, mask, _, embeds, _ = self.prepare_inputs_labels_for_multimodal(ids, None, attention_mask, None, None, images)
            finally:
                self._tls.feats_override = None
            if embeds is None:
                embeds = self.get_model().embed_tokens(ids.to(self.device))
                valid = None if attention_mask is None else attention_mask.bool()
            else:
                valid = self._tls.plan_mask if mask is None else mask.bool()
            # prefix reuse (reuse.PrefixCache): a finished request's sequence whose first rows are this request's first rows
            keys, reused = None, 0
            if self._prefix is not None and embeds.shape[0] == 1 and (valid is None or bool(valid.all())):
                keys = self._request_row_keys(ids, embeds.shape[1])
            if keys is not None:
                holder, n_common = self._prefix.take(keys, whole=self.exact_prefixes)
                if holder is not None:
                    p = min(n_common, embeds.shape[1] - 1)        # at least one row goes through the decoder: its logits pick the first token
                    if not self.exact_prefixes:
                        p -= p % 8                                 # the fused q|k|v epilogue wants pos0 % 8 == 0
                    if p >= self._prefix.min_rows and lib.lmx_seq_truncate(holder.seqs[0], p, stream_handle()) == 0:
                        cache, reused = holder, p
                        self._prefix.rows_reused += p
                    else:
                        holder.close()
            if cache is None:
                cache = LmxKVCache(self, 1)
            cache.row_keys, cache.reused_rows, cache.out_ref = keys, reused, None
            if reused:
                embeds = embeds[:, reused:]
                valid = None
            if sampling is not None:
                # the draw happens on the device (csrc/sampling.hip): temperature -> top-k -> top-p -> multinomial, keyed by a seed
                # taken from torch's CPU generator (so torch.manual_seed makes a request reproducible)
                temperature, top_p, top_k, seed = sampling
                check(lib.lmx_seq_set_sampling(cache.seqs[0], float(temperature), float(top_p if top_p is not None else 1.0), int(top_k or 0), int(seed)),
                      "lmx_seq_set_sampling")
            self._set_stop(cache.seqs[0], stop)          # before the prefill: its own pick (token 1) is tested too
            return {"cache": cache, "embeds": embeds, "valid": valid}
        except BaseException:
            if cache is not None:
                cache.close()
            raise

    def _request_row_keys(self, ids: torch.Tensor, T: int):
        """reuse.row_keys of the request just spliced on this thread (or of a text-only request), None if it cannot be keyed."""
        from .reuse import row_keys
        src = getattr(self._tls, "plan_src", None)
        if src is None:                                   # no image: the rows are the token ids
            k = ids.detach().cpu().numpy().astype(np.int64).reshape(-1)
            return k if len(k) == T and (k >= 0).all() else None
        hashes = getattr(self._tls, "image_hashes", None)
        if hashes is None or src.shape[0] != 1 or src.shape[1] != T:
            return None
        return row_keys(src[0], hashes, int(self._tls.plan_P))

    def _release_request_cache(self, cache: "LmxKVCache", out: Optional[Sequence[int]] = None) -> None:
        """End of a request: its sequence goes to the prefix cache — keyed by the prompt rows and the generated ids that have KV rows (all but the last
        one) — or back to the engine's pool."""
        keys = getattr(cache, "row_keys", None)
        if out is None:
            out = getattr(cache, "out_ref", None)
        pc = self._prefix
        if keys is None or pc is None or not cache.seqs:
            cache.close()
            return
        try:
            gen = np.asarray(list(out or [])[:-1], dtype=np.int64)
            full = np.concatenate([keys, gen]) if len(gen) else keys
            n = min(len(full), int(lib.lmx_seq_length(cache.seqs[0])))
            if n < pc.min_rows or (self.exact_prefixes and n != int(lib.lmx_seq_length(cache.seqs[0]))):
                cache.close()
                return
            cache.row_keys = None
            pc.put(full[:n], cache)
        except BaseException:  # noqa: BLE001
            cache.close()
            raise

    def _run_prepared(self, prepared: Sequence[dict], prefill_chunk: int = 0, return_logits: bool = False):
        """The collective-bearing half: the decoder prefill of prepared requests — one goes through lmx_prefill (same bits as generate()), several TOGETHER
        through lmx_prefill_batch (one GEMM per linear over the packed rows of all of them).  Every rank of a tensor-parallel group must call this with the
        same requests in the same order.  On failure the caches are the caller's to close."""
        if len(prepared) == 1:
            p = prepared[0]
            last = self._prefill_rows(p["cache"], p["embeds"], p["valid"], want_all=False, greedy=True, chunk=prefill_chunk)
            return last if return_logits else None
        packed = []
        for p in prepared:
            e, valid = p["embeds"][0], p["valid"]
            if valid is not None and not bool(valid[0].all()):
                e = e.index_select(0, torch.nonzero(valid[0].to(self.device), as_tuple=False).flatten())
            packed.append(e.to(self.dtype).contiguous())
        n = len(prepared)
        seqs = [p["cache"].seqs[0] for p in prepared]
        arr = (ctypes.c_void_p * n)(*[q.value if isinstance(q, ctypes.c_void_p) else q for q in seqs])
        eptr = (ctypes.c_void_p * n)(*[e.data_ptr() for e in packed])
        cnt = (ctypes.c_int32 * n)(*[int(e.shape[0]) for e in packed])
        check(lib.lmx_prefill_batch(self._h, arr, n, eptr, cnt, int(prefill_chunk) * n if prefill_chunk else 0, 1, stream_handle()), "lmx_prefill_batch")
        return None

    def _prefill_request(self, ids, images, attention_mask, sampling, prefill_chunk: int = 0, return_logits: bool = False, stop=None):
        """Image encode + splice + prefill of ONE request (ids [1, L]) into a fresh sequence; the first pick (argmax, or a draw when
        `sampling` = (temperature, top_p, top_k, seed) is given) is on the device when the stream gets there.  Shared by the request
        thread (generate) and the scheduler threads (batching.py, tp_serving.py)."""
        p = self._prepare_request(ids, images, attention_mask, sampling, stop)
        try:
            last = self._run_prepared([p], prefill_chunk, return_logits=return_logits)
            return (p["cache"], last) if return_logits else p["cache"]
        except BaseException:
            p["cache"].close()
            raise

    def _prefill_requests(self, reqs: Sequence[dict], prefill_chunk: int = 0) -> List["LmxKVCache"]:
        """Several requests prefilled TOGETHER (lmx_prefill_batch: one GEMM per linear over the packed rows of all of them).  reqs: dicts with ids [1, L],
        images, attention_mask, sampling (as _prefill_request takes them).  One request takes the single-sequence path (same bits as generate())."""
        prepared: List[dict] = []
        try:
            for r in reqs:
                prepared.append(self._prepare_request(r["ids"].to(self.device), r["images"], r["attention_mask"], r["sampling"], r.get("stop")))
            self._run_prepared(prepared, prefill_chunk)
            return [p["cache"] for p in prepared]
        except BaseException:
            for p in prepared:
                p["cache"].close()
            raise

    def _generate_one(self, ids, images, attention_mask, greedy, temperature, top_p, top_k, max_new_tokens, eos_set, streamer,
                      stopping_criteria, run_ahead, prefill_chunk) -> List[int]:
        if max_new_tokens <= 0:
            return []
        crit = list(stopping_criteria) if stopping_criteria is not None else []
        out: List[int] = []

        def make_emit(budget: int):
            def emit(tok: int) -> bool:
                out.append(tok)
                if streamer is not None:
                    streamer.put(torch.tensor([tok]))
                if tok in eos_set:
                    return True
                if crit:
                    full = torch.cat([ids.cpu(), torch.tensor([out], dtype=torch.long)], dim=1)
                    if any(c(full, None) for c in crit):
                        return True
                return len(out) >= budget
            return emit

        stop = self._stop_spec(eos_set, crit)           # the id rules go with the sequence to the device (lmx_seq_set_stop)
        batcher = self._batcher
        if batcher is not None and not prefill_chunk:
            prefill_chunk = self._batch_prefill_chunk
        if batcher is not None and (batcher.channel is not None or batcher.scheduler_prefill):
            # the scheduler thread prefills: under tensor parallelism because every call that carries a collective must be issued in an order the
            # leader broadcasts to the followers first (tp_serving.py); on one GPU (packed_prefill) because the requests waiting at that moment are
            # prefilled TOGETHER, one GEMM per linear over all their rows (lmx_prefill_batch).  The request thread hands the request over and waits
            sampling = None if greedy else (float(temperature), top_p, top_k, int(torch.randint(0, 2 ** 62, (1,)).item()))
            request = {"ids": ids.cpu(), "images": images, "attention_mask": None if attention_mask is None else attention_mask.cpu(),
                       "sampling": sampling, "prefill_chunk": int(prefill_chunk), "stop": stop, "out_ref": out}
            if getattr(batcher, "prepare_on_request_thread", False) and batcher.queued() < batcher.capacity:      # (a prepared request holds a sequence: bounded)
                # the rank-local half of the prefill here, on this request's own thread and stream (beside the running decode steps and the other requests'
                # prefills): image encode or feature-cache hit, splice, prefix-cache take.  The prefill thread then packs ready rows only
                prepared = self._prepare_request(ids.to(self.device), images, attention_mask, sampling, stop)
                request["prepared"], request["rows"] = prepared, int(prepared["embeds"].shape[1])
                # (from here the scheduler owns the prepared sequence: it closes it if the request never reaches a prefill)
            batcher.submit_request(request, make_emit, int(max_new_tokens))
            return out
        # With the batching scheduler on, image encode + prefill of concurrent requests run one at a time: k prefills sharing the GPU
        # all finish late (time to first token = k x one prefill for everybody), one after the other finishes the first after one.
        gate = self._prefill_gate if batcher is not None else None
        if gate is not None:
            gate.acquire()
        try:
            sampling = None if greedy else (float(temperature), top_p, top_k, self._draw_seed())
            cache = self._prefill_request(ids, images, attention_mask, sampling, prefill_chunk, stop=stop)
            seq = cache.seqs[0]
            if gate is not None:
                torch.cuda.current_stream(self.device).synchronize()      # the next request's prefill starts when this one is done
        finally:
            if gate is not None:
                gate.release()
        try:
            n_ctx = lib.lmx_seq_length(seq)
            budget = min(max_new_tokens, self.s_max - n_ctx)
            # A streamer wants every token as it is made.  Stopping criteria alone do not: they are evaluated per prefix on the ids read back in
            # run-ahead batches (same stop position as the reference's per-token check, mm_utils.py:94-107).  The id rules (EOS, keyword ids) are also
            # applied on the device by the pick itself, so no id exists past such a stop; only a TEXT-rule stop leaves ids behind it to drop
            interactive = streamer is not None
            emit = make_emit(budget)

            if batcher is not None:
                # continuous batching: this request's decode steps share the weight stream with every other live request
                host1 = (ctypes.c_int64 * 1)(); n1 = ctypes.c_int32(0)
                check(lib.lmx_seq_read_tokens(seq, host1, 1, ctypes.byref(n1), stream_handle()), "read_tokens")
                if not emit(int(host1[0])):
                    batcher.submit(seq, emit, room=budget - 1)
                return out
            host = (ctypes.c_int64 * (budget + 1))()
            n = ctypes.c_int32(0)
            done, consumed = False, 0
            # token 1 is the prefill's pick (argmax or draw); afterwards chain `ahead` steps on the device per host round trip.
            # Tokens produced past a stop are discarded (the cache is dropped with the sequence).
            produced = 1
            while True:
                check(lib.lmx_seq_read_tokens(seq, host, budget + 1, ctypes.byref(n), stream_handle()), "read_tokens")
                while consumed < min(n.value, produced) and not done:
                    done = emit(int(host[consumed])); consumed += 1
                if done or produced >= budget or n.value < produced:        # n < produced: the device-side rule stopped the sequence
                    break
                ahead = 1 if interactive else run_ahead
                ahead = max(1, min(ahead, budget - produced))
                check(lib.lmx_decode(self._h, seq, -1, ahead, None, 1, stream_handle()), "lmx_decode")
                produced += ahead
            return out
        finally:
            self._release_request_cache(cache, out)      # to the prefix cache (enable_reuse) or back to the pool
