"""Replay a recorded schedule of token ids through a model and dump logits.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR [--max-tokens N]

Input: one JSON line per step with `step` (its number), `entries` (each `id`, `tokens`: the request's next ids, `want`: indices into `tokens`) and `end` (ids of requests
that are over).  A step's entries form one batch: ids of new or continued requests go through the packed prefill in one call; entries that bring a single id to a running
request go through the decode batch.  Logits at the wanted indices are written to OUT/<step>.f32 as little-endian fp32 rows of `vocab` values, entries first, then `want`
in the order given; nothing is written for a step that wants none.  A request named in `end` returns its sequence to the pool.  Each step is acknowledged on standard
output by `done <step>`.

The family is chosen by config.json (registry.py); sequences, packed prefill, decode batch and kernels are those of generate()."""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict, List

import torch

from .batching import DecodeBatch
from .engine_lm import EngineCausalLM, LmxKVCache
from .registry import load_model

DECODE_ROWS = 256        # most sequences one decode batch holds


class TraceReplay:
    def __init__(self, model: EngineCausalLM):
        self.model = model
        self.live: Dict[str, LmxKVCache] = {}
        self._batch = None

    def _decode_batch(self, n: int) -> DecodeBatch:
        if self._batch is None or self._batch.capacity < n:
            if self._batch is not None:
                self._batch.close()
            cap = 1
            while cap < n:
                cap *= 2
            self._batch = DecodeBatch(self.model, cap)
        return self._batch

    def step(self, entries: List[dict]) -> torch.Tensor:
        """Run one step; logits [wanted, vocab] fp32 on the host, in order."""
        m = self.model
        order = [(e, w) for e in entries for w in e["want"]]
        fresh = {e["id"] for e in entries if e["id"] not in self.live}
        decode = [e for e in entries if e["id"] not in fresh and len(e["tokens"]) == 1]
        portion = [e for e in entries if not (e["id"] not in fresh and len(e["tokens"]) == 1) and e["tokens"]]
        rows: Dict[tuple, torch.Tensor] = {}
        for e in portion:
            if e["id"] in fresh:
                self.live[e["id"]] = LmxKVCache(m, 1)
        if portion:
            self._prefill(portion, rows)
        for i in range(0, len(decode), DECODE_ROWS):
            self._decode(decode[i:i + DECODE_ROWS], rows)
        V = m.config.vocab_size
        if not order:
            torch.cuda.current_stream(m.device).synchronize()
            return torch.empty((0, V))
        return torch.stack([rows[(e["id"], w)] for e, w in order])[:, :V].float().cpu()

    def _prefill(self, entries: List[dict], rows: Dict[tuple, torch.Tensor]) -> None:
        m = self.model
        embeds = m.get_model().embed_tokens(torch.tensor([t for e in entries for t in e["tokens"]], dtype=torch.long))
        parts = list(embeds.split([len(e["tokens"]) for e in entries]))
        wants = [sorted(set(e["want"])) for e in entries]
        logits = m.prefill_logits([self.live[e["id"]] for e in entries], parts, wants)
        for row, key in zip(logits, [(e["id"], r) for e, w in zip(entries, wants) for r in w]):
            rows[key] = row

    def _decode(self, entries: List[dict], rows: Dict[tuple, torch.Tensor]) -> None:
        m, n = self.model, len(entries)
        logits = torch.empty((n, m._vocab_cap), dtype=m.logits_dtype, device=m.device)
        self._decode_batch(n).step([self.live[e["id"]].seqs[0] for e in entries], [e["tokens"][0] for e in entries], 1, False, logits)
        for e, row in zip(entries, logits):
            rows[(e["id"], 0)] = row

    def end(self, request: str) -> None:
        cache = self.live.pop(request, None)
        if cache is not None:
            cache.close()

    def close(self) -> None:
        for r in list(self.live):
            self.end(r)
        if self._batch is not None:
            self._batch.close()
            self._batch = None


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a trace of token ids and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, default=0, help="most tokens the live requests hold together: capacity of a sequence's cache (0: the model's own)")
    a = ap.parse_args(argv)
    model = load_model(a.model, dtype=getattr(torch, a.dtype), max_position=a.max_tokens or None)
    replay = TraceReplay(model)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = replay.step(s["entries"])
        if logits.shape[0]:
            path = os.path.join(a.out, f"{s['step']}.f32")
            with open(path + ".part", "wb") as f:
                f.write(logits.contiguous().numpy().astype("<f4").tobytes())
            os.replace(path + ".part", path)
        for r in s.get("end", []):
            replay.end(r)
        print(f"done {s['step']}", flush=True)
    replay.close()
    return 0


if __name__ == "__main__":
    sys.exit(main())
