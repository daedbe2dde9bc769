"""The in-process inference engine — the Ollama replacement.

The reference worker shells out to an external Ollama daemon over HTTP
(reference: client/src/services/OllamaService.ts:97-284). Here the engine is
in-process: Llama-family models on PyTorch-ROCm with hand-written CDNA4
kernels (gridllm_amd.ops), a slot-based KV cache in HBM3E, hipGraph-captured
decode steps (bucketed batch sizes), and a full sampler. Tokens stream to a
callback — no per-token HTTP/JSON hop (SURVEY.md §3.3 hot-loop fix).
"""

from __future__ import annotations

import threading
import time
from contextlib import nullcontext as _nullctx

import numpy as np
from dataclasses import dataclass, field
from typing import Callable, Optional, Sequence

import torch

from gridllm_amd.config import EngineConfig
from gridllm_amd.engine import chat as chat_mod
from gridllm_amd.engine.sampler import SamplerState, sample
from gridllm_amd.engine.tokenizer import load_tokenizer
from gridllm_amd.models import model_class
from gridllm_amd.models.registry import resolve_spec
from gridllm_amd.parallel.tp import TPContext
from gridllm_amd.types import SamplingOptions
from gridllm_amd.utils.logging import get_logger

log = get_logger("engine")

# finer granularity in the serving range: a live batch of 192 must not
# pay a 256-wide padded graph replay (25% wasted weight reads)
_BUCKETS = (1, 2, 4, 8, 16, 24, 32, 48, 64, 96, 128, 160, 192, 224, 256,
            320, 384, 448, 512, 640, 768, 896, 1024)


@dataclass
class GenerationResult:
    text: str = ""
    token_ids: list[int] = field(default_factory=list)
    done_reason: str = "stop"
    prompt_eval_count: int = 0
    prompt_eval_duration: int = 0   # ns
    eval_count: int = 0
    eval_duration: int = 0          # ns
    total_duration: int = 0
    cancelled: bool = False


@dataclass
class _Row:
    slot: int
    state: SamplerState
    decoder: object
    on_token: Optional[Callable[[str, bool], None]]
    cancel: Optional[threading.Event]
    stops: list[str]
    max_new: int
    result: GenerationResult
    last_token: int = 0
    fast: bool = False             # no constraint/stops/penalties: _emit
                                   # takes the short path (hot at b1024)
    text_tail: str = ""            # pending window for stop-sequence matching
    force_cancel: bool = False     # TP: rank-0-synchronized cancel decision
    done: bool = False
    t_start_ns: int = 0            # wall clock at admission
    t_decode_ns: int = 0           # wall clock when prefill+first token done
    cur_len: int = 0               # storage length in the KV slot
    constraint: object = None      # grammar automaton (format="json")
    todo: list[int] = field(default_factory=list)   # prompt tokens not run yet
                                   # (models with mixed steps)


class InferenceEngine:
    def __init__(self, cfg: Optional[EngineConfig] = None,
                 tp: Optional[TPContext] = None):
        self.cfg = cfg or EngineConfig()
        self.tp = tp or TPContext()
        dev = self.cfg.device
        if dev == "auto":
            dev = "cuda:0" if torch.cuda.is_available() else "cpu"
        self.device = torch.device(dev)
        self.is_gpu = self.device.type == "cuda"
        if self.is_gpu and self.tp.size > 1:
            torch.cuda.set_device(self.device)
        dtype = self.cfg.dtype
        if not self.is_gpu and dtype != "fp32":
            dtype = "fp32"          # CPU reference path runs fp32
        if self.cfg.max_batch_size < 1:
            raise ValueError("max_batch_size must be at least 1")
        spec = resolve_spec(self.cfg.model, self.cfg.weights_path,
                            self.cfg.max_seq_len)
        t0 = time.monotonic_ns()
        import glob as _glob
        import os as _os
        have_weights = bool(self.cfg.weights_path) and bool(_glob.glob(
            _os.path.join(self.cfg.weights_path, "*.safetensors")))
        cls = model_class(spec)
        # a model with mixed steps runs portions of prompts beside decoded
        # tokens; its KV memory is a pool of tokens, not of full-length slots
        self.mixed = getattr(cls, "supports_mixed", False)
        self.shift_ok = (self.cfg.context_shift
                         and getattr(cls, "supports_shift", True))
        extra = {"kv_tokens": self.cfg.kv_tokens,
                 "random_init": not have_weights} if self.mixed else {}
        # +1 scratch slot for hipGraph warmup/padding rows
        self.model = cls(spec, device=str(self.device), dtype=dtype,
                         tp=self.tp, seed=self.cfg.seed,
                         kv_slots=self.cfg.max_batch_size + 1,
                         max_seq=self.cfg.max_seq_len, **extra)
        if self.cfg.weights_path:
            if have_weights:
                n = self.model.load_safetensors(self.cfg.weights_path)
                log.performance("weights loaded", tensors=n,
                                path=self.cfg.weights_path)
            else:
                log.logger.warning(
                    "weights_path %r has no .safetensors; random init",
                    self.cfg.weights_path)
        if self.is_gpu and dtype == "bf16":
            self.model.interleave_gateup()   # fused-SwiGLU projection layout
        self.load_duration = time.monotonic_ns() - t0
        self.spec = spec
        self.tokenizer = load_tokenizer(self.cfg.weights_path, spec.vocab)
        # the scratch slot absorbs hipGraph warmup + padding-row traffic and
        # must never be handed to a real request (determinism bug otherwise)
        self._scratch_slot = self.cfg.max_batch_size  # last slot
        self.model.cache.reserve(self._scratch_slot)
        # device-resident index for the per-step scratch reset: a host
        # scalar write (`seq_lens[i] = 0`) stalls ~0.5 ms against a busy
        # stream; index_fill_ with this cached index enqueues instead
        self._scratch_idx = torch.tensor([self._scratch_slot],
                                         dtype=torch.int64,
                                         device=self.device)
        self._graphs: dict[int, tuple] = {}
        self._graph_pool = None
        # admission prefill runs on its own HIP stream: prefill is
        # MFMA-bound while decode replay is HBM-bound, and at
        # prompt≈num_predict the workload is ~half prefill FLOPs —
        # serializing them on one stream left the decode stream idle for
        # the whole prefill pass (the engine-vs-serving 2x gap)
        self._pf_stream = torch.cuda.Stream(device=self.device) \
            if self.is_gpu else None
        import os as _os
        self._no_emit_text = \
            _os.environ.get("GRIDLLM_NO_EMIT_TEXT", "0") == "1"
        from gridllm_amd.engine.sampler import SlotSampler
        self.sampler = SlotSampler(self.cfg.max_batch_size + 1, self.device)
        if self.is_gpu and self.cfg.autotune:
            from gridllm_amd.ops.autotune import tune_model_shapes
            buckets = [b for b in _BUCKETS if b <= self.cfg.max_batch_size]
            if self.cfg.max_batch_size not in buckets:
                buckets.append(self._bucket(self.cfg.max_batch_size))
            tune_model_shapes(self.model, sorted(set(buckets)))
        self._lock = threading.Lock()
        if self.is_gpu:
            self.precapture_graphs()
        log.performance("engine ready", model=spec.name,
                        params=spec.params, device=str(self.device),
                        tp=self.tp.size, load_ms=self.load_duration // 1_000_000)

    # ------------------------------------------------------------------ sync

    def _sync(self) -> None:
        if self.is_gpu:
            torch.cuda.synchronize(self.device)

    # -------------------------------------------------------------- hipGraph

    def _graph_ok(self) -> bool:
        if not (self.is_gpu and self.cfg.use_hipgraph):
            return False
        if self.tp.size == 1:
            return True
        # TP decode is hipGraph-captured too: the
        # per-layer RCCL all-reduces are captured with the step. Needs the
        # nccl(=RCCL) backend — gloo collectives are host ops and cannot
        # be captured (the tp2-on-one-GPU CI configuration).
        import os as _os
        return (self.tp.backend == "nccl"
                and _os.environ.get("GRIDLLM_TP_GRAPH", "1") != "0")

    def _bucket(self, b: int) -> int:
        for x in _BUCKETS:
            if x >= b:
                return x
        return b

    def _ensure_graph(self, bucket: int):
        if bucket in self._graphs:
            return self._graphs[bucket]
        if self._pf_stream is not None:
            # a mid-serving capture must not race an in-flight side-stream
            # admission prefill (capture invalidates concurrent work)
            self._pf_stream.synchronize()
        tokens = torch.zeros(bucket, dtype=torch.int64, device=self.device)
        slots = torch.full((bucket,), self._scratch_slot, dtype=torch.int32,
                           device=self.device)
        # warmup on a side stream (required before capture)
        s = torch.cuda.Stream()
        s.wait_stream(torch.cuda.current_stream())
        with torch.cuda.stream(s):
            for _ in range(2):
                self.model.forward_decode(tokens, slots)
                # reset BETWEEN iterations: each warmup advances the scratch
                # slot by `bucket` positions, and at bucket >= max_seq the
                # second pass would write past the slot's KV region (the
                # b=1024 x max_seq=1024 GPU fault)
                self.model.cache.seq_lens[self._scratch_slot] = 0
        torch.cuda.current_stream().wait_stream(s)
        g = torch.cuda.CUDAGraph()
        # ONE shared memory pool for every bucket graph: private per-graph
        # pools totalled 49.7 GB at max_batch 1536 (23 buckets) and OOM'd
        # the 288 GB card (gpurun_out/r02n_serving_c1536.log). Sharing is
        # safe under the capture-largest-first discipline (engine init
        # captures descending; a replay never outgrows the pool's high-
        # water mark set by the largest capture).
        if self._graph_pool is None:
            self._graph_pool = torch.cuda.graph_pool_handle()
        with torch.cuda.graph(g, pool=self._graph_pool):
            out = self.model.forward_decode(tokens, slots)
        self.model.cache.seq_lens[self._scratch_slot] = 0
        self._graphs[bucket] = (g, tokens, slots, out)
        log.performance("hipGraph captured", bucket=bucket)
        return self._graphs[bucket]

    def precapture_graphs(self) -> None:
        """Capture every bucket graph <= max_batch_size, LARGEST FIRST,
        into the shared pool (lazy capture order would let a later,
        larger bucket outgrow the pool)."""
        if not self._graph_ok():
            return
        try:
            for b in sorted((x for x in _BUCKETS
                             if x <= self.cfg.max_batch_size),
                            reverse=True):
                self._ensure_graph(b)
        except Exception:  # noqa: BLE001 — degrade loudly to eager
            log.logger.exception(
                "hipGraph precapture failed — running eager decode")
            self.cfg.use_hipgraph = False
            self._graphs.clear()

    def _decode_step(self, token_ids: list[int], slot_ids: list[int],
                     slots_t: "Optional[torch.Tensor]" = None
                     ) -> torch.Tensor:
        """Run one decode step for rows (token, slot). Returns logits [B, V].
        slots_t: optional prebuilt device int32 slot tensor (callers that
        also sample by slot share ONE upload per step)."""
        b = len(token_ids)
        self.model.cache.prepare_decode(slot_ids)
        if self._graph_ok():
            bucket = self._bucket(b)
            try:
                g, tbuf, sbuf, out = self._ensure_graph(bucket)
            except Exception:  # noqa: BLE001
                # graph capture failed (e.g. an RCCL build without
                # collective-capture support at tp>1): degrade LOUDLY to
                # eager — a capture crash at scale-out time would take the
                # whole TP group down instead
                log.logger.exception(
                    "hipGraph capture failed — falling back to eager decode")
                self.cfg.use_hipgraph = False
                g = None
            if g is not None:
                tbuf[:b] = torch.as_tensor(token_ids, dtype=torch.int64,
                                           device=self.device)
                if b < bucket:
                    tbuf[b:] = 0
                    sbuf[b:] = self._scratch_slot
                    # keep the scratch slot from overflowing across replays
                    self.model.cache.seq_lens[self._scratch_slot] = 0
                if slots_t is not None:
                    sbuf[:b] = slots_t
                else:
                    sbuf[:b] = torch.as_tensor(slot_ids, dtype=torch.int32,
                                               device=self.device)
                g.replay()
                return out[:b]
        tokens = torch.as_tensor(token_ids, dtype=torch.int64, device=self.device)
        slots = slots_t if slots_t is not None else torch.as_tensor(
            slot_ids, dtype=torch.int32, device=self.device)
        return self.model.forward_decode(tokens, slots)

    # -------------------------------------------------------- mixed steps
    # (models with supports_mixed: the step that generation runs on, and the
    #  way to feed given tokens, e.g. to replay a trace)

    def open_sequence(self, tokens: int = 0) -> int:
        """A fresh sequence; `tokens` > 0 sets memory aside for that many,
        otherwise it grows while there is some. Returns its slot."""
        with self._lock:
            return self.model.cache.alloc(tokens)

    def close_sequence(self, slot: int) -> None:
        with self._lock:
            self.model.cache.free(slot)

    def run_step(self, entries: Sequence[tuple]) -> torch.Tensor:
        """Run one batch of (slot, token ids, wanted places) and return the
        logits f32 [wanted, vocab] in that order."""
        with self._lock:
            return self._run_step(entries)

    def _run_step(self, entries: Sequence[tuple]) -> torch.Tensor:
        if not self.mixed:
            raise NotImplementedError(
                f"{self.spec.name} has no mixed steps")
        lens = self.model.cache.lens
        if all(len(ids) == 1 and lens[sl] > 0 for sl, ids, _ in entries):
            # nothing but decoding: the captured step
            for _, ids, _ in entries:
                if not 0 <= ids[0] < self.spec.vocab:
                    raise ValueError("token id outside of the vocabulary")
            logits = self._decode_step([ids[0] for _, ids, _ in entries],
                                       [sl for sl, _, _ in entries])
            if all(list(w) == [0] for _, _, w in entries):
                return logits
            return logits[[i for i, e in enumerate(entries) for _ in e[2]]]
        return self.model.forward_step(entries)

    def _mixed_step(self, active: list["_Row"]) -> list["_Row"]:
        """One step in which some rows still have prompt tokens to run: the
        others decode their next token beside as many prompt tokens, in order
        of admission, as the step's budget takes. Returns the rows still
        running."""
        for r in active:
            if r.todo and self._cancelled(r):
                r.result.done_reason = "cancelled"
                r.result.cancelled = True
                self._retire(r)
        active = [r for r in active if not r.done]
        left = self.cfg.prefill_chunk
        entries, emitting = [], []
        for r in active:
            if not r.todo:
                entries.append((r.slot, [r.last_token], [0]))
                emitting.append(r)
                r.cur_len += 1
                continue
            part = r.todo[:left]
            if not part:
                continue
            left -= len(part)
            r.todo = r.todo[len(part):]
            entries.append((r.slot, part, [] if r.todo else [len(part) - 1]))
            if not r.todo:
                emitting.append(r)
        if not entries:
            return active
        logits = self._run_step(entries)
        if not emitting:
            return active
        slots = self.model.up.upload(
            np.asarray([r.slot for r in emitting], dtype=np.int64))
        toks = self._sample_batch(logits, emitting, slots)
        t1 = time.monotonic_ns()
        for r, tok in zip(emitting, toks):
            first = r.t_decode_ns == 0
            if first:
                r.result.prompt_eval_duration = t1 - r.t_start_ns
                r.t_decode_ns = t1
            if not (self._emit(r, tok) and (r.max_new > 1 or not first)):
                self._retire(r)
        return [r for r in active if not r.done]

    # ------------------------------------------------------------- sampling

    def _sample_batch(self, logits: torch.Tensor,
                      rows: Sequence[_Row],
                      slots_t: "Optional[torch.Tensor]" = None) -> list[int]:
        """Batched sampling; vectorized for the common uniform cases.
        With slots_t (device int64 slot ids) the per-slot device-resident
        sampler runs — zero per-step H2D (see sampler.SlotSampler)."""
        states = [r.state for r in rows]
        for i, r in enumerate(rows):
            c = getattr(r, "constraint", None)   # tolerate row shims
            if c is not None:
                self._apply_constraint_mask(logits[i], c)
        if all(s.greedy for s in states):
            return logits.argmax(dim=-1).tolist()
        if slots_t is not None:
            return self.sampler.sample(logits, rows, slots_t)
        from gridllm_amd.engine.sampler import (BatchPlan,
                                                sample_batch_vectorized)
        plan = getattr(self, "_sampler_plan", None)
        if plan is None:
            plan = self._sampler_plan = BatchPlan()
        return sample_batch_vectorized(logits, states, plan)

    def _apply_constraint_mask(self, row_logits: torch.Tensor,
                               constraint) -> None:
        """Mask row logits to the automaton's legal next bytes (+EOS when a
        complete value has been emitted). Byte tokenizer: ids 0..255 are
        raw bytes. In-place; no host sync. HF tokenizers dispatch to
        token-level lazy masking (constraints.mask_logits_token_level)."""
        if hasattr(self.tokenizer, "token_bytes"):
            from gridllm_amd.engine.constraints import \
                mask_logits_token_level
            mask_logits_token_level(row_logits, constraint, self.tokenizer,
                                    self.tokenizer.eos_id)
            return
        allowed, eos_ok = constraint.allowed()
        idx = list(allowed)
        if eos_ok:
            idx.append(self.tokenizer.eos_id)
        keep = torch.full_like(row_logits, float("-inf"))
        ix = torch.tensor(idx, dtype=torch.long, device=row_logits.device)
        keep[ix] = row_logits[ix]
        row_logits.copy_(keep)

    # ------------------------------------------------------------ main loop

    def generate(self, prompt: str, options: Optional[dict] = None,
                 on_token: Optional[Callable[[str, bool], None]] = None,
                 cancel: Optional[threading.Event] = None,
                 raw_stops: Optional[list[str]] = None) -> GenerationResult:
        return self.generate_batch([(prompt, options or {})],
                                   on_tokens=[on_token], cancels=[cancel],
                                   extra_stops=raw_stops)[0]

    def chat(self, messages: list[dict], options: Optional[dict] = None,
             on_token: Optional[Callable[[str, bool], None]] = None,
             cancel: Optional[threading.Event] = None,
             think: bool = False) -> GenerationResult:
        fam = chat_mod.family_of(self.spec.name)
        prompt = chat_mod.render_chat(messages, think=think, family=fam)
        return self.generate(prompt, options, on_token, cancel,
                             raw_stops=chat_mod.chat_stops(fam))

    def embed(self, inputs: list[str]) -> list[list[float]]:
        out: list[list[float]] = []
        for i0 in range(0, len(inputs), 16):      # bound KV-slot pressure
            chunk = inputs[i0:i0 + 16]
            with self._lock:
                token_lists = [torch.as_tensor(self._encode(t),
                                               dtype=torch.int64,
                                               device=self.device)
                               for t in chunk]
                nslots = min(len(chunk),
                             max(1, self.model.cache.n_free))
                hiddens = []
                for j0 in range(0, len(chunk), nslots):
                    part = token_lists[j0:j0 + nslots]
                    slots = [self.model.cache.alloc(len(t)) for t in part]
                    try:
                        _, h = self.model.forward_prefill_batch(
                            part, slots, return_hidden=True)
                        hiddens.append(h)
                    finally:
                        for sl in slots:
                            self.model.cache.free(sl)
                hidden = torch.cat(hiddens)
            for vec in hidden.detach().cpu():
                n = vec.norm()
                out.append((vec / n if n > 0 else vec).tolist())
        return out

    def _encode(self, prompt: str) -> list[int]:
        ids = self.tokenizer.encode(prompt)
        limit = self.model.max_seq - 8
        if len(ids) > limit:
            ids = ids[-limit:]
        if not ids:
            ids = [0]
        return ids

    def generate_batch(self, requests: list[tuple[str, dict]],
                       on_tokens: Optional[list] = None,
                       cancels: Optional[list] = None,
                       extra_stops: Optional[list[str]] = None
                       ) -> list[GenerationResult]:
        """Prefill each request, then batched decode until all complete."""
        with self._lock:
            return self._generate_batch(requests, on_tokens, cancels,
                                        extra_stops)

    def _generate_batch(self, requests, on_tokens, cancels, extra_stops
                        ) -> list[GenerationResult]:
        n = len(requests)
        on_tokens = on_tokens or [None] * n
        cancels = cancels or [None] * n
        rows = self._start_rows(
            [(prompt, opts_d, on_tokens[i], cancels[i], extra_stops)
             for i, (prompt, opts_d) in enumerate(requests)])
        active = [r for r in rows if not r.done]
        try:
            while active:
                active = self._step_rows(active)
        except Exception:
            self.abort_rows(active, locked=True)   # no slot leak on failure
            raise
        return [r.result for r in rows]

    # -------------------------------------------------- row-stepping API
    # (continuous batching: the batcher admits rows into a live decode
    #  loop; generate_batch above is the run-to-completion wrapper used
    #  by the TP lockstep path and tests)

    def start_row(self, prompt: str, opts_d: dict,
                  on_token: Optional[Callable[[str, bool], None]] = None,
                  cancel: Optional[threading.Event] = None,
                  extra_stops: Optional[list[str]] = None) -> _Row:
        with self._lock:
            return self._start_rows([(prompt, opts_d, on_token, cancel,
                                      extra_stops)])[0]

    def start_rows(self, items: list[tuple]) -> list["_Row"]:
        """Admit a BATCH of requests: one concatenated prefill pass (GEMMs
        at M = sum of prompt lengths instead of per-prompt launches), then
        batched first-token sampling. items: (prompt, opts_d, on_token,
        cancel, extra_stops) tuples."""
        with self._lock:
            return self._start_rows(items)

    def step_rows(self, rows: list["_Row"]) -> list["_Row"]:
        with self._lock:
            return self._step_rows(rows)

    def start_rows_async(self, items: list[tuple]) -> list["_Row"]:
        """Pipelined admission: prefill + first-token sampling LAUNCH but
        never sync — the admission's GPU wait stalled the decode pipeline
        ~10% at c1024 (round-2 profile: 124 admission syncs x ~20 ms).
        First tokens are emitted by the NEXT collect_step (the submit
        that follows attaches this batch). Caller guarantees no
        constraint/penalty rows and a running pipeline (batcher checks)."""
        with self._lock:
            # Dedicated prefill stream: the whole admission pass (uploads,
            # prefill kernels, first-token sample, D2H) overlaps the
            # decode graph replays in flight on the main stream — the
            # slots are fresh (no step references them until the first
            # post-admission submit, which waits on ev below). Decode is
            # HBM-bound and prefill MFMA-bound, so they genuinely share
            # the chip rather than time-slicing it.
            pf = self._pf_stream
            ctx = torch.cuda.stream(pf) if pf is not None else _nullctx()
            with ctx:
                rows, logits, slots_t = self._prefill_rows(items)
                try:
                    ids_dev = self.sampler.sample_ids(logits, rows, slots_t)
                except Exception:
                    self.abort_rows(rows, locked=True)
                    raise
                b = len(rows)
                ev = None
                if self.is_gpu:
                    ih = self._pinned_admit(b)
                    ih[:b].copy_(ids_dev, non_blocking=True)
                    ev = torch.cuda.Event()
                    ev.record()
                else:
                    ih = ids_dev
            self._admit_pending = {
                "rows": rows, "ids_dev": ids_dev, "ids_host": ih,
                "ev": ev,
                "pos": {id(r): i for i, r in enumerate(rows)}}
            return rows

    def _start_rows(self, items: list[tuple]) -> list["_Row"]:
        if self.mixed:
            # nothing runs yet: the prompts go through the next steps
            rows, id_lists = self._make_rows(items)
            for row, ids in zip(rows, id_lists):
                row.todo = list(ids)
            self.sampler.admit(rows, self.spec.vocab)
            return rows
        rows, logits, slots_t = self._prefill_rows(items)
        try:
            toks = self._sample_batch(logits, rows, slots_t)  # syncs
        except Exception:
            self.abort_rows(rows, locked=True)
            raise
        t1 = time.monotonic_ns()
        per = (t1 - rows[0].t_start_ns) // max(1, len(rows)) if rows else 0
        for row, tok in zip(rows, toks):
            row.result.prompt_eval_duration = per
            row.t_decode_ns = t1
            if not (self._emit(row, tok) and row.max_new > 1):
                self._retire(row)
        return rows

    def _make_rows(self, items: list[tuple]):
        """Rows with a cache slot each, and their prompts' token ids."""
        t0 = time.monotonic_ns()
        rows: list[_Row] = []
        id_lists: list[list[int]] = []
        slots: list[int] = []
        try:
            for prompt, opts_d, on_token, cancel, extra_stops in items:
                opts = SamplingOptions.from_dict(opts_d)
                ids = self._encode(prompt)
                if opts.num_ctx:
                    ids = ids[-max(16, min(opts.num_ctx,
                                           self.model.max_seq - 8)):]
                id_lists.append(ids)
                stops = list(opts.stop or [])
                if extra_stops:
                    stops += extra_stops
                # Ollama default (num_predict -1/unset): generate until EOS
                # or the context fills — NOT a fixed cap (round-1 verdict
                # gap 4: a generate without num_predict must not truncate
                # where the reference stack would not)
                max_new = opts.num_predict \
                    if opts.num_predict and opts.num_predict > 0 \
                    else (1 << 30)
                if self.shift_ok:
                    # the KV window slides, so generation is bounded by the
                    # rope table (original absolute positions), not max_seq
                    max_new = min(max_new,
                                  self.model.rope_len - len(ids) - 1)
                else:
                    max_new = min(max_new,
                                  self.model.max_seq - len(ids) - 1)
                constraint = None
                if (getattr(self.tokenizer, "BOS", None) is not None
                        or hasattr(self.tokenizer, "token_bytes")):
                    # byte tokenizer -> exact byte-grammar masking;
                    # HF tokenizer -> token-level lazy masking over the
                    # same byte automaton (constraints.py). A dict format
                    # is a JSON schema (Ollama contract) -> the
                    # schema-directed automaton (schema_constraints.py)
                    if opts.format == "json":
                        from gridllm_amd.engine.constraints import \
                            JsonByteConstraint
                        constraint = JsonByteConstraint()
                    elif isinstance(opts.format, dict):
                        from gridllm_amd.engine.schema_constraints import \
                            JsonSchemaByteConstraint
                        constraint = JsonSchemaByteConstraint(opts.format)
                # tokens the slot may come to hold (a pipelined retire runs
                # one decode step too many)
                slot = self.model.cache.alloc(
                    min(self.model.max_seq, len(ids) + max_new + 1))
                slots.append(slot)
                row = _Row(slot=slot,
                           state=SamplerState.create(opts, self.device),
                           decoder=self.tokenizer.decode_stream(),
                           on_token=on_token, cancel=cancel,
                           stops=stops, max_new=max_new,
                           result=GenerationResult(),
                           t_start_ns=t0, cur_len=len(ids),
                           constraint=constraint)
                row.result.prompt_eval_count = len(ids)
                row.fast = (constraint is None and not stops
                            and not row.state.has_penalty)
                rows.append(row)
        except Exception:
            for sl in slots:          # release what this batch allocated
                self.model.cache.free(sl)
            raise
        return rows, id_lists

    def _prefill_rows(self, items: list[tuple]):
        rows, id_lists = self._make_rows(items)
        slots = [r.slot for r in rows]
        try:
            # ONE pinned upload for every prompt's ids (one blocking H2D
            # per prompt measured ~1.5 ms each against a busy stream)
            all_ids = self.model.up.upload(np.concatenate(
                [np.asarray(x, dtype=np.int64) for x in id_lists]))
            token_lists = list(torch.split(all_ids,
                                           [len(x) for x in id_lists]))
            if len(rows) == 1:
                logits = self.model.forward_prefill(token_lists[0],
                                                    slots[0]).unsqueeze(0)
            else:
                logits = self.model.forward_prefill_batch(token_lists, slots)
            self._sync_cancel(rows)
            self.sampler.admit(rows, self.spec.vocab)
            slots_t = self.model.up.upload(
                np.asarray(slots, dtype=np.int64))
        except Exception:
            # prefill failure: release every slot this batch allocated
            # or capacity leaks permanently
            self.abort_rows(rows, locked=True)
            raise
        return rows, logits, slots_t

    def abort_rows(self, rows: Sequence["_Row"], locked: bool = False) -> None:
        """Free the KV slots of rows that have not retired (step/prefill
        failure cleanup). Safe to call with already-retired rows: _retire
        sets done and frees exactly once."""
        if not locked:
            with self._lock:
                return self.abort_rows(rows, locked=True)
        for r in rows:
            if not r.done:
                r.done = True
                self.model.cache.free(r.slot)

    def _step_rows(self, active: list["_Row"]) -> list["_Row"]:
        """One batched decode step; returns the rows still running."""
        if any(r.todo for r in active):
            return self._mixed_step(active)
        if self.shift_ok:
            for r in active:
                if r.cur_len >= self.model.max_seq:
                    r.cur_len = self.model.shift_slot(r.slot)
        token_ids = [r.last_token for r in active]
        slot_ids = [r.slot for r in active]
        # one slot upload per step, shared by decode (int32 view) and the
        # per-slot sampler (int64)
        slots64 = torch.as_tensor(slot_ids, dtype=torch.int64,
                                  device=self.device)
        logits = self._decode_step(token_ids, slot_ids,
                                   slots_t=slots64.to(torch.int32))
        next_ids = self._sample_batch(logits, active, slots64)
        self._sync_cancel(active)
        still: list[_Row] = []
        for r, tok in zip(active, next_ids):
            r.cur_len += 1
            if self._emit(r, tok):
                still.append(r)
            else:
                self._retire(r)
        return still

    # ------------------------------------------------ pipelined stepping
    # The synchronous loop serializes: GPU step -> host sync -> per-token
    # bookkeeping -> next step; at serving batch sizes the host segment is
    # 30-50% of the step. The pipelined path submits step N with step
    # N-1's sampled ids STILL ON DEVICE (a gather feeds the next graph
    # replay), then processes N-1's ids on the host while N runs. Costs:
    # retires land one step late (one wasted decode step per finishing
    # row); rows with grammar constraints, sampling penalties, or at the
    # context boundary take the synchronous path; TP stays synchronous
    # (the follower mirror steps in lockstep).

    def pipeline_ok(self, rows: Sequence["_Row"]) -> bool:
        if self.tp.enabled:
            return False
        for r in rows:
            if r.todo or r.constraint is not None or r.state.has_penalty:
                return False
            if r.cur_len + 2 > self.model.max_seq:
                return False
        return True

    def _pinned(self, n: int) -> torch.Tensor:
        """Reusable pinned host buffers (ring of 2: one in flight, one
        being collected)."""
        cache = getattr(self, "_pin_ring", None)
        if cache is None:
            cache = self._pin_ring = {}
        ring = cache.setdefault(n, [None, None, 0])
        i = ring[2] = (ring[2] + 1) % 2
        if ring[i] is None:
            ring[i] = torch.empty(n, dtype=torch.int64, pin_memory=True)
        return ring[i]

    def _pinned_admit(self, n: int) -> torch.Tensor:
        """Pinned readback buffers for ASYNC ADMISSIONS — a ring separate
        from _pinned: an admission interleaved between two same-size steps
        breaks the step ring's strict alternation, and the next step's
        enqueued D2H can land in the buffer a collect is still reading
        (silent token corruption when b_admit == b_step)."""
        cache = getattr(self, "_pin_admit_ring", None)
        if cache is None:
            cache = self._pin_admit_ring = {}
        ring = cache.setdefault(n, [None, None, 0])
        i = ring[2] = (ring[2] + 1) % 2
        if ring[i] is None:
            ring[i] = torch.empty(n, dtype=torch.int64, pin_memory=True)
        return ring[i]

    def _pinned_stage(self, n: int) -> torch.Tensor:
        """Pinned upload staging (ring of 2 — the previous upload may
        still be in flight when the next composition change happens)."""
        cache = getattr(self, "_stage_ring", None)
        if cache is None:
            cache = self._stage_ring = {}
        ring = cache.setdefault(n, [None, None, 0])
        i = ring[2] = (ring[2] + 1) % 2
        if ring[i] is None:
            ring[i] = torch.empty(n, dtype=torch.int64, pin_memory=True)
        return ring[i]

    def submit_step(self, rows: list["_Row"], prev=None):
        """Launch one decode step WITHOUT waiting for its result.
        Token sources: rows present in `prev` gather their token from
        prev's on-device ids; others (new admissions, sync-stepped rows)
        use their host-known last_token. Returns an inflight handle for
        collect_step. Caller ensures pipeline_ok(rows)."""
        with self._lock:
            import numpy as np
            b = len(rows)
            if self.shift_ok:
                for r in rows:
                    if r.cur_len >= self.model.max_seq:
                        r.cur_len = self.model.shift_slot(r.slot)
            ap = getattr(self, "_admit_pending", None)
            self._admit_pending = None
            if ap is not None and ap.get("ev") is not None:
                # first step that includes the admitted rows: order the
                # main stream after the side-stream prefill, and tell the
                # allocator ids_dev is consumed here (torch.where below)
                cur = torch.cuda.current_stream()
                cur.wait_event(ap["ev"])
                ap["ids_dev"].record_stream(cur)
            same = (ap is None and prev is not None
                    and len(prev["rows"]) == b
                    and all(a is c for a, c in zip(prev["rows"], rows)))
            if same:
                # steady state (no admit/retire since the last step): the
                # previous step's on-device ids feed straight in, slot
                # tensors are reused — ZERO host->device traffic
                tokens_dev = prev["ids_dev"]
                slots64 = prev["slots64"]
                slots32 = prev["slots32"]
            else:
                src = np.full(b, -1, dtype=np.int64)
                src2 = np.full(b, -1, dtype=np.int64)
                host_tok = np.zeros(b, dtype=np.int64)
                slots_np = np.zeros(b, dtype=np.int64)
                pos = prev["pos"] if prev is not None else {}
                apos = ap["pos"] if ap is not None else {}
                for i, r in enumerate(rows):
                    src[i] = pos.get(id(r), -1)
                    src2[i] = apos.get(id(r), -1)
                    host_tok[i] = r.last_token
                    slots_np[i] = r.slot
                # pinned staging + non_blocking: a pageable .to(device)
                # enqueues BEHIND the in-flight step and blocks the host
                # on it (~1.5 ms/step measured) — the exact stall the
                # pipeline exists to remove
                if self.is_gpu:
                    stage = self._pinned_stage(4 * b).view(4, b)
                    stage.numpy()[:] = np.stack(
                        [src, host_tok, slots_np, src2])
                    up = torch.empty(4, b, dtype=torch.int64,
                                     device=self.device)
                    up.copy_(stage, non_blocking=True)
                else:
                    up = torch.from_numpy(
                        np.stack([src, host_tok, slots_np, src2]))
                tokens_dev = up[1]
                if prev is not None:
                    tokens_dev = torch.where(
                        up[0] >= 0,
                        prev["ids_dev"][up[0].clamp(min=0)], tokens_dev)
                if ap is not None:
                    # async-admitted rows: first token straight from the
                    # admission's on-device sample
                    tokens_dev = torch.where(
                        up[3] >= 0,
                        ap["ids_dev"][up[3].clamp(min=0)], tokens_dev)
                slots64 = up[2]
                slots32 = slots64.to(torch.int32)
            if self.mixed:
                self.model.cache.prepare_decode([r.slot for r in rows])
            if self._graph_ok():
                bucket = self._bucket(b)
                try:
                    g, tbuf, sbuf, out = self._ensure_graph(bucket)
                except Exception:  # noqa: BLE001
                    log.logger.exception(
                        "hipGraph capture failed — eager decode")
                    self.cfg.use_hipgraph = False
                    g = None
                if g is not None:
                    tbuf[:b] = tokens_dev
                    if b < bucket:
                        tbuf[b:] = 0
                        sbuf[b:] = self._scratch_slot
                        self.model.cache.seq_lens.index_fill_(
                            0, self._scratch_idx, 0)
                    sbuf[:b] = slots32
                    g.replay()
                    logits = out[:b]
                else:
                    logits = self.model.forward_decode(tokens_dev, slots32)
            else:
                logits = self.model.forward_decode(tokens_dev, slots32)
            ids_dev = self.sampler.sample_ids(logits, rows, slots64)
            if self.is_gpu:
                ids_host = self._pinned(b)
                ids_host[:b].copy_(ids_dev, non_blocking=True)
                ev = torch.cuda.Event()
                ev.record()
            else:
                ids_host, ev = ids_dev, None
            for r in rows:
                r.cur_len += 1          # the step appended to the KV slot
            free_after = getattr(self, "_deferred_free", [])
            self._deferred_free = []
            return {"rows": rows, "ids_dev": ids_dev, "ids_host": ids_host,
                    "ev": ev, "pos": {id(r): i for i, r in enumerate(rows)},
                    "slots64": slots64, "slots32": slots32,
                    "free_after": free_after, "admit": ap}

    def collect_step(self, inflight) -> None:
        """Wait for an inflight step's sampled ids and run the per-token
        bookkeeping (emit/stop/EOS/retire). Slots retired here stay
        allocated until the NEXT collect (they were already inside the
        following in-flight step)."""
        with self._lock:
            ev = inflight["ev"]
            if ev is not None:
                ev.synchronize()
            ap = inflight.get("admit")
            if ap is not None:
                # async admission batch: its prefill + first-token sample
                # ran BEFORE this step on the same stream, so this step's
                # event covers its pinned copy too
                ids0 = ap["ids_host"][:len(ap["rows"])].tolist()
                t1 = time.monotonic_ns()
                for r, tok in zip(ap["rows"], ids0):
                    if r.done:
                        continue
                    # includes ~one overlapped decode step (no sync point
                    # exists to time the prefill alone on this path)
                    r.result.prompt_eval_duration = t1 - r.t_start_ns
                    r.t_decode_ns = t1
                    if not (self._emit(r, int(tok)) and r.max_new > 1):
                        self._retire(r, defer_free=True)
            ids = inflight["ids_host"][:len(inflight["rows"])].tolist()
            for r, tok in zip(inflight["rows"], ids):
                if r.done:
                    continue            # retired while this step flew
                if not self._emit(r, int(tok)):
                    self._retire(r, defer_free=True)
            for sl in inflight["free_after"]:
                self.model.cache.free(sl)

    def flush_admit(self) -> None:
        """Resolve a pending async admission WITHOUT a following pipelined
        step (the batcher fell back to the synchronous path, e.g. a live
        row reached the context boundary): sync the stream and emit the
        first tokens so the rows have valid last_token state."""
        with self._lock:
            ap = getattr(self, "_admit_pending", None)
            self._admit_pending = None
            if ap is None:
                return
            self._sync()
            ids0 = ap["ids_host"][:len(ap["rows"])].tolist()
            t1 = time.monotonic_ns()
            for r, tok in zip(ap["rows"], ids0):
                if r.done:
                    continue
                r.result.prompt_eval_duration = t1 - r.t_start_ns
                r.t_decode_ns = t1
                if not (self._emit(r, int(tok)) and r.max_new > 1):
                    self._retire(r)
            return

    def flush_deferred(self) -> None:
        """Free retire-deferred slots once NO step is in flight (pipeline
        drain / fallback to the synchronous path)."""
        with self._lock:
            for sl in getattr(self, "_deferred_free", []):
                self.model.cache.free(sl)
            self._deferred_free = []

    def _sync_cancel(self, rows: Sequence[_Row]) -> None:
        """Under TP every rank must retire the same rows at the same step, or
        the next collective deadlocks (SURVEY.md §7 hard-part 5). Rank 0 owns
        the cancel events; the decision is broadcast and applied via
        force_cancel on all ranks (including rank 0 — its own event could
        flip between broadcast and emit otherwise)."""
        if not self.tp.enabled:
            return
        # host tensor over the gloo CONTROL group: no GPU sync, and the
        # compute stream (possibly mid-graph-replay) is never touched
        flags = torch.tensor(
            [1 if (r.cancel is not None and r.cancel.is_set()) else 0
             for r in rows], dtype=torch.int32)
        self.tp.broadcast_cpu(flags, src=0)
        for r, f in zip(rows, flags.tolist()):
            if f:
                r.force_cancel = True

    def _cancelled(self, row: _Row) -> bool:
        if self.tp.enabled:
            return row.force_cancel
        return row.cancel is not None and row.cancel.is_set()

    def _emit(self, row: _Row, tok: int) -> bool:
        """Record a sampled token; returns False when the row is finished."""
        res = row.result
        res.token_ids.append(tok)
        res.eval_count += 1
        row.last_token = tok
        if row.fast:
            # hot path (no constraint/stops/penalties — the serving bulk):
            # ~2.4 ms/step of this loop runs on the decode thread at b1024
            row.state.draws += 1       # keeps slot re-admission keys exact
            if self._cancelled(row):
                res.done_reason = "cancelled"
                res.cancelled = True
                return False
            if tok == self.tokenizer.eos_id:
                res.done_reason = "stop"
                return False
            if not self._no_emit_text:
                piece = row.decoder.push(tok)
                if piece:
                    res.text += piece
                    if row.on_token:
                        row.on_token(piece, False)
            if res.eval_count >= row.max_new:
                res.done_reason = "length"
                return False
            return True
        row.state.observe(tok, self.spec.vocab)
        if row.constraint is not None:
            try:
                if hasattr(self.tokenizer, "token_bytes"):
                    bs = self.tokenizer.token_bytes(tok)
                    if bs:
                        row.constraint.push_bytes(bs)
                elif 0 <= tok < 256:
                    row.constraint.push(tok)
            except ValueError:
                res.done_reason = "stop"   # automaton refused (shouldn't
                return False               # happen with masking in place)
        if self._cancelled(row):
            res.done_reason = "cancelled"
            res.cancelled = True
            return False
        if tok == self.tokenizer.eos_id:
            res.done_reason = "stop"
            return False
        if self._no_emit_text:
            # diagnostic mode (GRIDLLM_NO_EMIT_TEXT=1): skip per-token
            # text decode/stream emission to measure its end-to-end cost;
            # final text still assembled at retire from token_ids
            if res.eval_count >= row.max_new:
                res.done_reason = "length"
                return False
            return True
        piece = row.decoder.push(tok)
        if piece:
            row.text_tail += piece
            emit_now = row.text_tail
            if row.stops:
                for st in row.stops:
                    idx = row.text_tail.find(st)
                    if idx >= 0:
                        final = row.text_tail[:idx]
                        if final:
                            res.text += final
                            if row.on_token:
                                row.on_token(final, False)
                        res.done_reason = "stop"
                        row.text_tail = ""
                        return False
                # hold back a window that could begin a stop sequence
                hold = max(len(s) for s in row.stops) - 1
                emit_now = row.text_tail[:-hold] if hold > 0 else row.text_tail
                row.text_tail = row.text_tail[len(emit_now):]
            else:
                row.text_tail = ""
            if emit_now:
                res.text += emit_now
                if row.on_token:
                    row.on_token(emit_now, False)
        if res.eval_count >= row.max_new:
            res.done_reason = "length"
            return False
        return True

    def _retire(self, row: _Row, defer_free: bool = False) -> None:
        if self._no_emit_text:
            final = self.tokenizer.decode(row.result.token_ids)
        else:
            tail = row.decoder.flush() if hasattr(row.decoder, "flush") \
                else ""
            final = row.text_tail + tail
        if final and not row.result.cancelled:
            row.result.text += final
            if row.on_token:
                row.on_token(final, False)
        row.text_tail = ""
        t_end = time.monotonic_ns()
        row.result.eval_duration = max(0, t_end - row.t_decode_ns)
        row.result.total_duration = t_end - row.t_start_ns
        row.done = True
        if row.on_token:
            row.on_token("", True)
        if defer_free:
            # pipelined retire: the slot is still referenced by the step
            # currently in flight — free only after that step collects
            if not hasattr(self, "_deferred_free"):
                self._deferred_free = []
            self._deferred_free.append(row.slot)
        else:
            self.model.cache.free(row.slot)

    # ------------------------------------------------------------- metadata

    def model_names(self) -> list[str]:
        from gridllm_amd.models.registry import names_for
        try:
            return names_for(self.spec.name)
        except KeyError:
            return [self.spec.name]

    def stats(self) -> dict:
        return {
            "model": self.spec.name,
            "params": self.spec.params,
            "device": str(self.device),
            "tp": self.tp.size,
            "kv_slots_free": self.model.cache.n_free,
            "max_seq": self.model.max_seq,
        }
