"""Engine: schedules sequences over a registered model and its caches, so that generation runs (and its throughput can be
measured) on token ids, without a tokenizer.

What it mirrors of the reference's engine:
  * the metadata the model runner hands to the layers (nanovllm/engine/model_runner.py:120-180): int32 cu_seqlens,
    slot_mapping, context_lens, block_tables padded with -1;
  * the scheduling policy (nanovllm/engine/scheduler.py:25-59): prefill first, limited by
    max_num_batched_tokens / max_num_seqs, otherwise one decode step for every running sequence.
  * optional HIP-graph replay of the decode forward for bucketed batch sizes with static input buffers,
    slot_mapping padded with -1 and context_lens with 0 (model_runner.py:189-206, 216-251).
Beyond the reference:
  * models come from a registry (models/): Qwen3, and decoders put together from a list of layers.  A model says whether it
    needs pages, state slots or both; the cache manager hands them out per sequence.
  * a step may bring portions: any number of next tokens per sequence, portions of prompts beside single decoded tokens in
    one batch (run_portions).  With chunked_prefill the scheduler makes such batches itself: every running sequence decodes
    one token and what is left of max_num_batched_tokens goes to prompts, cut where the budget ends.
  * with graphs captured, generate() does not wait for a step's tokens before it issues
    the next step.  Which sequences run, their lengths, slots and block tables depend only on token counts, so
    the host prepares step t+1 while the GPU works on step t; the sampled tokens stay on the device (one row
    per sequence, gathered as the next step's input ids) and are read back once at the end.  The reference
    reads them back every step (model_runner.py:212), which leaves the GPU idle while the host schedules.
Not mirrored: prefix caching, preemption (the cache is sized so it never triggers), tensor parallelism,
the tokenizer.

Every tensor op goes through a mops backend looked up by name, so the Qwen3 model runs on the `hip`
backend and on any other registered one.
"""
from __future__ import annotations

import time
from collections import deque
from dataclasses import dataclass, field

import torch

from . import mops  # noqa: F401  (binds the operator backend)
from .cache import CacheManager
from .models import load_config, model_class
from .models.qwen3 import Qwen3Shape
from .weights import CheckpointWeights, RandomWeights

BLOCK_SIZE = 256


@dataclass
class Sequence:
    token_ids: list
    max_tokens: int
    temperature: float
    num_prompt_tokens: int = 0
    block_table: list = field(default_factory=list)
    state_slot: int = -1
    num_cached: int = 0    # tokens whose keys, values and state the device holds
    row: int = -1      # pipelined generation: this sequence's row in the device-side last-token table
    filled: int = 0    # pipelined generation: completion tokens whose values have been read back

    def __post_init__(self):
        self.num_prompt_tokens = len(self.token_ids)

    def __len__(self):
        return len(self.token_ids)

    @property
    def num_completion_tokens(self):
        return len(self.token_ids) - self.num_prompt_tokens


class Engine:
    def __init__(self, shape=None, backend: str = "hip", num_blocks: int = 2560, seed: int = 0,
                 max_num_batched_tokens: int = 16384, max_num_seqs: int = 512, device="cuda:0", weights=None,
                 dtype=torch.bfloat16, block_size: int = BLOCK_SIZE, num_state_slots: int = None, max_model_len: int = 32768,
                 chunked_prefill: bool = False):
        """shape: a configuration of a registered model (default: Qwen3-0.6B).  weights: a source with take() (default:
        seeded random tensors of `dtype`).  max_model_len bounds the positions of models without a bound of their own."""
        self.shape = shape if shape is not None else Qwen3Shape()
        self.dev = torch.device(device)
        self.backend = backend
        self.max_num_batched_tokens = max_num_batched_tokens
        self.max_num_seqs = max_num_seqs
        self.chunked_prefill = chunked_prefill
        cls = model_class(self.shape)
        self.dtype = weights.dtype if weights is not None else dtype
        if self.dtype not in cls.dtypes:
            raise ValueError(f"{cls.__name__} does not run in {self.dtype}")
        pages, slots = cls.needs(self.shape)
        self.cache = CacheManager(num_blocks, block_size, (max_num_seqs if num_state_slots is None else num_state_slots) if slots else 0,
                                  self.dev, pages=pages, slots=slots)
        self.block_size = block_size
        self.num_blocks = num_blocks
        self.model = cls(self.shape, weights if weights is not None else RandomWeights(seed, self.dtype, self.dev), self.cache,
                         backend=backend, max_model_len=max_model_len)
        self.op_linear, self.op_sampler_forward = self.model.op_linear, self.model.op_sampler_forward
        self.waiting: deque = deque()
        self.running: deque = deque()
        self.graphs = {}
        self.graph_bs = []
        # pipelined generation (see the module docstring): last sampled token per sequence row; row 0
        # takes the writes of padding rows
        self.pipelined = True
        self.last_tok = torch.zeros(max_num_seqs + 1, dtype=torch.int64, device=self.dev)
        self.free_rows = deque(range(1, max_num_seqs + 1))
        self.unit_temps = torch.ones(max_num_seqs, dtype=torch.float32, device=self.dev)
        self._sampler_checked = False
        self.capture_stream = None

    @classmethod
    def from_pretrained(cls, folder, dtype=torch.bfloat16, device="cuda:0", **options):
        """An engine on the model of a folder: config.json chooses the model class, *.safetensors hold its weights."""
        config = load_config(folder)
        if dtype not in model_class(config).dtypes:
            raise ValueError(f"{model_class(config).__name__} does not run in {dtype}")
        return cls(config, device=device, weights=CheckpointWeights(folder, dtype, device), **options)

    # what callers of the engine reach through it
    @property
    def free_blocks(self):
        return self.cache.free_blocks

    @property
    def kv_cache(self):
        return self.model.kv_cache

    @property
    def op_qk_norm_rope_store(self):
        return self.model.op_qk_norm_rope_store

    @property
    def use_fused_qk(self):
        return self.model.use_fused_qk

    @use_fused_qk.setter
    def use_fused_qk(self, on):
        self.model.use_fused_qk = on

    @property
    def share_decode_plan(self):
        return self.model.share_decode_plan

    @share_decode_plan.setter
    def share_decode_plan(self, on):
        self.model.share_decode_plan = on

    def forward(self, input_ids, positions, ctx):
        return self.model.forward(input_ids, positions, ctx)

    def _check_sampler_ignores_temperature(self):
        """Pipelined generation hands the sampler unit temperatures (the per-sequence ones would cost a gather per step).
        That is only right while the backend's sampler is greedy, as the reference's is (mops/torch/ops.py:37-43 with
        the sampling line commented out): checked once, on random logits, before the first pipelined run."""
        if self._sampler_checked:
            return
        g = torch.Generator(device=self.dev).manual_seed(1234)
        logits = torch.randn((8, 4096), generator=g, device=self.dev, dtype=torch.float32).to(torch.bfloat16)
        hot = torch.full((8,), 0.3, dtype=torch.float32, device=self.dev)
        a = self.op_sampler_forward(logits, self.unit_temps[:8])
        b = self.op_sampler_forward(logits, hot)
        if not torch.equal(a, b):
            raise RuntimeError(f"the {self.backend} backend's sampler depends on the temperature: pipelined generation "
                               "passes unit temperatures and would sample differently; set engine.pipelined = False")
        self._sampler_checked = True

    # ------------------------------------------------------------------ HIP graphs for decode
    @torch.inference_mode()
    def capture_decode_graphs(self, max_bs: int = 256, max_model_len: int = 4096, smallest_first: bool = False):
        """Captures the decode forward (embedding .. final norm) once per batch-size bucket.  Replays
        read their inputs from static buffers; rows beyond the live batch carry slot -1 / length 0,
        which store_kvcache skips and paged decode answers with zeros.  The order of the captures does not matter
        (smallest_first exists for the test of that)."""
        max_blocks = (max_model_len + self.block_size - 1) // self.block_size
        dev = self.dev
        self.g_ids = torch.zeros(max_bs, dtype=torch.int64, device=dev)
        self.g_i64 = torch.zeros((2, max_bs), dtype=torch.int64, device=dev)    # int64 copies of rows and positions
        self.g_rows64, self.g_pos = self.g_i64[0], self.g_i64[1]
        # the int32 inputs are views of one buffer, so that one host-to-device copy can fill them all:
        # [sequence rows | positions | slots | lengths | state slots | block tables]
        self.g_meta = torch.empty(max_bs * (5 + max_blocks), dtype=torch.int32, device=dev)
        self.g_rows, self.g_pos32 = self.g_meta[:max_bs], self.g_meta[max_bs:2 * max_bs]
        self.g_slots, self.g_lens = self.g_meta[2 * max_bs:3 * max_bs], self.g_meta[3 * max_bs:4 * max_bs]
        self.g_states = self.g_meta[4 * max_bs:5 * max_bs]
        self.g_tables = self.g_meta[5 * max_bs:].view(max_bs, max_blocks)
        self.g_rows.zero_()
        self.g_pos32.zero_()
        self.g_slots.fill_(-1)
        self.g_lens.zero_()
        self.g_states.fill_(-1)
        self.g_tables.fill_(-1)
        self.g_out = torch.zeros((max_bs, self.model.hidden), dtype=self.dtype, device=dev)
        self.graph_bs = [b for b in (1, 2, 4, 8) if b <= max_bs] + list(range(16, max_bs + 1, 16))
        # Every bucket is captured on one stream of our own.  The ops keep their scratch buffers per stream, and
        # the graphs hold those addresses: sizing the scratch for the largest bucket on that stream before the
        # first capture means no capture, in whatever order, allocates or moves it.
        # The stream stays alive with the engine: the scratch is keyed by the stream's handle, and a handle that went back
        # to torch's pool could be handed to unrelated eager work, which would then share the graphs' scratch.
        capture_stream = self.capture_stream = self.capture_stream or torch.cuda.Stream(dev)
        with torch.cuda.stream(capture_stream):
            self.model.reserve_graph_scratch(max_bs, max_blocks)
        pool = None
        for bs in (self.graph_bs if smallest_first else reversed(self.graph_bs)):
            ctx = dict(is_prefill=False, slot_mapping=self.g_slots[:bs], context_lens=self.g_lens[:bs],
                       block_tables=self.g_tables[:bs], hidden_only=True, n_decode=bs, state_slots=self.g_states[:bs],
                       starts=self.g_pos32[:bs], positions32=self.g_pos32[:bs], token_context=self.g_lens[:bs], token_seq=None,
                       cu_seqlens=None)
            graph = torch.cuda.CUDAGraph()
            self.g_out[:bs] = self.forward(self.g_ids[:bs], self.g_pos[:bs], ctx)      # warm-up outside capture
            torch.cuda.synchronize(dev)
            with torch.cuda.graph(graph, pool, stream=capture_stream):
                self.g_out[:bs] = self.forward(self.g_ids[:bs], self.g_pos[:bs], ctx)
            if pool is None:
                pool = graph.pool()
            self.graphs[bs] = graph
        torch.cuda.synchronize(dev)

    @torch.inference_mode()
    def _decode_replay(self, ids, pos, ctx):
        bs = ids.numel()
        bucket = next(b for b in self.graph_bs if b >= bs)
        self.g_ids[:bs] = ids
        self.g_pos[:bs] = pos
        self.g_pos32[:bs] = ctx["positions32"]
        self.g_states.fill_(-1)
        if ctx["state_slots"] is not None:
            self.g_states[:bs] = ctx["state_slots"]
        self.g_slots.fill_(-1)
        self.g_slots[:bs] = ctx["slot_mapping"]
        self.g_lens.zero_()
        self.g_lens[:bs] = ctx["context_lens"]
        self.g_tables[:bs, : ctx["block_tables"].size(1)] = ctx["block_tables"]
        self.graphs[bucket].replay()
        # the lm head runs on the bucket's row count, like the captured layers: GEMM solutions are chosen per shape
        return self.model.logits(self.g_out[:bucket])[:bs]

    # ------------------------------------------------------------------ metadata (model_runner.py:120-187)
    def _to_dev(self, data, dtype):
        return torch.tensor(data, dtype=dtype, pin_memory=True).to(self.dev, non_blocking=True)

    def _block_tables(self, seqs):
        width = max(1, max(len(q.block_table) for q in seqs))
        return self._to_dev([q.block_table + [-1] * (width - len(q.block_table)) for q in seqs], torch.int32)

    def _slots(self, q, begin, end):
        """Cache rows of the tokens [begin, end) of a sequence; -1 where the model keeps no pages."""
        if not self.cache.uses_pages:
            return [-1] * (end - begin)
        bs, table = self.block_size, q.block_table
        return [table[t // bs] * bs + t % bs for t in range(begin, end)]

    def _last_slots(self, seqs):
        """Cache row of the last token of each sequence (the whole list at once: a decode step pays for every call)."""
        if not self.cache.uses_pages:
            return [-1] * len(seqs)
        bs = self.block_size
        return [q.block_table[-1] * bs + (len(q.token_ids) - 1) % bs for q in seqs]

    def _prepare_portions(self, seqs, counts):
        """Batch of the next counts[i] tokens of seqs[i] behind the num_cached tokens of earlier steps.  Layers run single
        tokens, short and long portions on different kernels, each on a run of the batch: callers sort by count."""
        n_decode = 0
        while n_decode < len(seqs) and counts[n_decode] == 1:
            n_decode += 1
        ids, pos, token_seq, slots, cu, starts = [], [], [], [], [0], []
        for i, (q, n) in enumerate(zip(seqs, counts)):
            begin = q.num_cached
            ids.extend(q.token_ids[begin:begin + n])
            pos.extend(range(begin, begin + n))
            token_seq.extend([i] * n)
            slots.extend(self._slots(q, begin, begin + n))
            cu.append(cu[-1] + n)
            starts.append(begin)
        lens = [s + n for s, n in zip(starts, counts)]
        cu_ctx = [0]
        for n in lens:
            cu_ctx.append(cu_ctx[-1] + n)
        p32 = self._to_dev(pos, torch.int32)
        portions = token_seq[n_decode:]
        ctx = dict(is_prefill=True, has_prefix=any(starts), max_seqlen=max(counts), max_context=max(lens), n_decode=n_decode,
                   seq_counts=list(counts), seq_starts=starts,
                   cu_seqlens=self._to_dev(cu, torch.int32), cu_context=self._to_dev(cu_ctx, torch.int32),
                   starts=self._to_dev(starts, torch.int32), context_lens=self._to_dev(lens, torch.int32),
                   state_slots=self._to_dev([q.state_slot for q in seqs], torch.int32),
                   token_seq=self._to_dev(token_seq, torch.int32), positions32=p32, token_context=p32 + 1,
                   portion_cu=self._to_dev([c - n_decode for c in cu[n_decode:]], torch.int32),
                   portion_token_seq=self._to_dev([i - n_decode for i in portions], torch.int32),
                   slot_mapping=self._to_dev(slots, torch.int32), block_tables=self._block_tables(seqs))
        return self._to_dev(ids, torch.int64), self._to_dev(pos, torch.int64), ctx

    def _prepare_prefill(self, seqs):
        """Whole sequences from their first token on."""
        for q in seqs:
            q.num_cached = 0
        return self._prepare_portions(seqs, [len(q) for q in seqs])

    def _prepare_decode(self, seqs):
        ids = [q.token_ids[-1] for q in seqs]
        pos = [len(q) - 1 for q in seqs]
        slots = self._last_slots(seqs)
        p32 = self._to_dev(pos, torch.int32)
        lens = self._to_dev([len(q) for q in seqs], torch.int32)
        ctx = dict(is_prefill=False, slot_mapping=self._to_dev(slots, torch.int32), context_lens=lens,
                   block_tables=self._block_tables(seqs), n_decode=len(seqs), starts=p32, positions32=p32, token_context=lens,
                   token_seq=None, cu_seqlens=None,
                   state_slots=self._to_dev([q.state_slot for q in seqs], torch.int32) if self.cache.uses_slots else None)
        return self._to_dev(ids, torch.int64), self._to_dev(pos, torch.int64), ctx

    @torch.inference_mode()
    def run_portions(self, portions):
        """One step on a mixed batch.  portions: (sequence, its next token ids, places among them whose logits are wanted);
        the tokens are appended to the sequence.  Returns the logits [wanted, vocab] in the order of the portions and of their
        places, or None when nothing is wanted."""
        for q, tokens, _ in portions:
            q.token_ids.extend(tokens[max(0, len(q) - q.num_cached):])
            self._check_length(q, q.num_cached + len(tokens))
            self.cache.hold(q, q.num_cached + len(tokens))
        order = sorted(range(len(portions)), key=lambda i: len(portions[i][1]))      # stable
        seqs, counts = [portions[i][0] for i in order], [len(portions[i][1]) for i in order]
        first = {}
        at = 0
        for i, n in zip(order, counts):
            first[i] = at
            at += n
        rows = [first[i] + w for i, (_, _, want) in enumerate(portions) for w in want]
        ids, pos, ctx = self._prepare_portions(seqs, counts)
        ctx["logit_rows"] = self._to_dev(rows, torch.int64)
        if not rows:
            ctx["hidden_only"] = True
        out = self.model.forward(ids, pos, ctx)
        for q, n in zip(seqs, counts):
            q.num_cached += n
        return out if rows else None

    # ------------------------------------------------------------------ scheduling (scheduler.py:25-72)
    def _check_length(self, q, n_tokens):
        if n_tokens > self.model.max_positions:
            raise ValueError(f"a sequence of {n_tokens} tokens exceeds the {self.model.max_positions} positions of this engine")

    def open_sequence(self):
        """A sequence without tokens, for callers that drive run_portions themselves."""
        return Sequence([], 0, 1.0)

    def close_sequence(self, q):
        self.cache.release(q)

    def add_request(self, token_ids, max_tokens, temperature=0.6):
        q = Sequence(list(token_ids), max_tokens, temperature)
        self._check_length(q, len(q) + max_tokens)
        self.waiting.append(q)

    def _schedule(self):
        batch, tokens = [], 0
        while self.waiting and len(batch) < self.max_num_seqs:
            q = self.waiting[0]
            if tokens + len(q) > self.max_num_batched_tokens or not self.cache.can_hold(q, len(q)):
                break
            self.cache.hold(q, len(q))
            tokens += len(q)
            self.waiting.popleft()
            self.running.append(q)
            batch.append(q)
        if batch:
            return sorted(batch, key=len), True
        batch = list(self.running)[: self.max_num_seqs]
        for q in batch:   # the token about to be written may open a new block
            self.cache.hold(q, len(q))
        return batch, False

    def _schedule_mixed(self):
        """(sequence, number of its next tokens) for one step: a token of every sequence that decodes, then prompts - those
        already begun first - as far as max_num_batched_tokens goes.  A prompt is admitted when its pages are free."""
        budget, batch = self.max_num_batched_tokens, []
        live = list(self.running)[: self.max_num_seqs]
        for q in (q for q in live if len(q) - q.num_cached == 1):
            if budget:
                self.cache.hold(q, len(q))
                batch.append((q, 1))
                budget -= 1
        for q in (q for q in live if len(q) - q.num_cached > 1):
            n = min(budget, len(q) - q.num_cached)
            if n:
                batch.append((q, n))
                budget -= n
        while self.waiting and budget and len(self.running) < self.max_num_seqs and self.cache.can_hold(self.waiting[0], len(self.waiting[0])):
            q = self.waiting.popleft()
            self.cache.hold(q, len(q))
            self.running.append(q)
            n = min(budget, len(q))
            batch.append((q, n))
            budget -= n
        return batch

    def _finish(self, seqs, tokens):
        """Appends one sampled token per sequence and releases what is complete; returns the finished ones."""
        finished = []
        for q, t in zip(seqs, tokens):
            q.token_ids.append(t)
            if q.num_completion_tokens >= q.max_tokens:
                finished.append(q)
        for q in finished:
            self.running.remove(q)
            self.cache.release(q)
        return finished

    @torch.inference_mode()
    def step(self):
        """One step of the scheduler; returns (sequences, whether prompts ran, finished sequences)."""
        if self.chunked_prefill:
            batch = self._schedule_mixed()
            done = [(q, n) for q, n in batch if q.num_cached + n == len(q)]
            has_prompts = any(q.num_cached < q.num_prompt_tokens for q, _ in batch)
            logits = self.run_portions([(q, q.token_ids[q.num_cached:q.num_cached + n], [n - 1] if q.num_cached + n == len(q) else [])
                                        for q, n in batch])
            seqs = [q for q, _ in done]
            tokens = []
            if seqs:
                tokens = self.op_sampler_forward(logits, self._to_dev([q.temperature for q in seqs], torch.float32)).tolist()
            return [q for q, _ in batch], has_prompts, self._finish(seqs, tokens)
        seqs, is_prefill = self._schedule()
        ids, pos, ctx = self._prepare_prefill(seqs) if is_prefill else self._prepare_decode(seqs)
        temps = self._to_dev([q.temperature for q in seqs], torch.float32)
        if not is_prefill and self.graphs and len(seqs) <= self.graph_bs[-1] and ctx["block_tables"].size(1) <= self.g_tables.size(1):
            logits = self._decode_replay(ids, pos, ctx)
        else:
            logits = self.forward(ids, pos, ctx)
        for q in seqs:
            q.num_cached = len(q)
        tokens = self.op_sampler_forward(logits, temps).tolist()     # the only device->host sync of a step
        return seqs, is_prefill, self._finish(seqs, tokens)

    @torch.inference_mode()
    def _generate_pipelined(self, stats):
        """Runs until no sequence is waiting or running without reading a token back in between."""
        import numpy as np
        self._check_sampler_ignores_temperature()
        dev = self.dev
        n, max_blocks = self.g_ids.numel(), self.g_tables.size(1)
        depth = 8                                  # steps the host may be ahead of the GPU
        staging = [torch.empty(self.g_meta.numel(), dtype=torch.int32, pin_memory=True) for _ in range(depth)]
        staged = [None] * depth                    # event: the copy out of that staging buffer has run
        hist_rows = 2048
        hist = torch.empty((hist_rows, self.max_num_seqs), dtype=torch.int64, device=dev)
        steps = []                                 # (history row, sequences, is_prefill, end-of-step event)
        mark = torch.cuda.Event(enable_timing=True)
        mark.record()

        def drain():
            nonlocal mark
            if not steps:
                return
            torch.cuda.synchronize(dev)
            host = hist[:len(steps)].cpu()
            prev = mark
            for h, seqs, is_prefill, ev in steps:
                row = host[h].tolist()
                for j, q in enumerate(seqs):
                    q.token_ids[q.num_prompt_tokens + q.filled] = row[j]
                    q.filled += 1
                stats["prefill_s" if is_prefill else "decode_s"] += prev.elapsed_time(ev) * 1e-3
                prev = ev
            mark = prev
            steps.clear()

        it = 0
        while self.waiting or self.running:
            if len(steps) == hist_rows:
                drain()
            seqs, is_prefill = self._schedule()
            bs = len(seqs)
            graphable = (not is_prefill and bs <= self.graph_bs[-1]
                         and max(len(q.block_table) for q in seqs) <= max_blocks)
            if is_prefill:
                if len(self.free_rows) < bs:     # more sequences in flight than rows so far: grow the table
                    old = self.last_tok.numel()
                    self.last_tok = torch.cat((self.last_tok, torch.zeros(max(bs, old), dtype=torch.int64, device=dev)))
                    self.free_rows.extend(range(old, self.last_tok.numel()))
                for q in seqs:
                    q.row = self.free_rows.popleft()
                ids, pos, ctx = self._prepare_prefill(seqs)
                logits = self.forward(ids, pos, ctx)
                rows = self._to_dev([q.row for q in seqs], torch.int64)
            elif graphable:
                slot = it % depth
                it += 1
                if staged[slot] is not None:
                    staged[slot].synchronize()
                a = staging[slot].numpy()
                a[:2 * n] = 0
                a[2 * n:3 * n] = -1
                a[3 * n:4 * n] = 0
                a[4 * n:] = -1                       # state slots and block tables
                a[:bs] = [q.row for q in seqs]
                a[n:n + bs] = [len(q) - 1 for q in seqs]
                a[2 * n:2 * n + bs] = self._last_slots(seqs)
                a[3 * n:3 * n + bs] = [len(q) for q in seqs]
                if self.cache.uses_slots:
                    a[4 * n:4 * n + bs] = [q.state_slot for q in seqs]
                tab = a[5 * n:].reshape(n, max_blocks)
                for j, q in enumerate(seqs):
                    tab[j, :len(q.block_table)] = q.block_table
                self.g_meta.copy_(staging[slot], non_blocking=True)
                staged[slot] = torch.cuda.Event()
                staged[slot].record()
                bucket = next(b for b in self.graph_bs if b >= bs)
                self.g_i64.copy_(self.g_meta[:2 * n].view(2, n))
                torch.index_select(self.last_tok, 0, self.g_rows64[:bucket], out=self.g_ids[:bucket])
                self.graphs[bucket].replay()
                logits = self.model.logits(self.g_out[:bucket])[:bs]
                rows = self.g_rows64[:bs]
            else:                                   # a batch no graph covers: this step runs the stepwise way
                drain()
                ids, pos, ctx = self._prepare_decode(seqs)
                logits = self.forward(ids, pos, ctx)
                rows = self._to_dev([q.row for q in seqs], torch.int64)
            tok = self.op_sampler_forward(logits, self.unit_temps[:bs])   # greedy: the temperature does not move the argmax
            self.last_tok.index_copy_(0, rows, tok)
            hist[len(steps), :bs] = tok
            ev = torch.cuda.Event(enable_timing=True)
            ev.record()
            steps.append((len(steps), list(seqs), is_prefill, ev))
            for q in seqs:
                q.token_ids.append(-1)              # value pending; only the count matters to the scheduler
                if q.num_completion_tokens >= q.max_tokens:
                    self.running.remove(q)
                    self.cache.release(q)
                    self.free_rows.append(q.row)
                    q.row = -1
            if is_prefill:
                stats["prefill_steps"] += 1
                stats["prefill_tokens"] += sum(len(q) - 1 for q in seqs)
            else:
                stats["decode_steps"] += 1
                stats["decode_tokens"] += bs
        drain()

    def generate(self, prompts, max_tokens, temperature=0.6):
        """prompts: list of token-id lists; max_tokens: int or list.  Returns (completions, stats)."""
        if isinstance(max_tokens, int):
            max_tokens = [max_tokens] * len(prompts)
        order = []
        for p, m in zip(prompts, max_tokens):
            self.add_request(p, m, temperature)
            order.append(self.waiting[-1])
        stats = dict(prefill_steps=0, decode_steps=0, prefill_tokens=0, decode_tokens=0, prefill_s=0.0, decode_s=0.0)
        torch.cuda.synchronize(self.dev)
        t_all = time.perf_counter()
        if self.graphs and self.pipelined and not self.chunked_prefill:
            self._generate_pipelined(stats)
        while self.waiting or self.running:     # stepwise: every step's tokens are read back before the next
            t0 = time.perf_counter()
            cached = sum(q.num_cached for q in self.running)
            seqs, is_prefill, _ = self.step()
            dt = time.perf_counter() - t0
            if is_prefill:
                stats["prefill_steps"] += 1
                stats["prefill_tokens"] += sum(q.num_cached for q in seqs) - cached if self.chunked_prefill else sum(len(q) - 1 for q in seqs)
                stats["prefill_s"] += dt
            else:
                stats["decode_steps"] += 1
                stats["decode_tokens"] += len(seqs)
                stats["decode_s"] += dt
        stats["total_s"] = time.perf_counter() - t_all
        return [q.token_ids[q.num_prompt_tokens:] for q in order], stats
