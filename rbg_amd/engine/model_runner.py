"""Model runner — builds kernel batches and executes model steps.

Owns the device, model, KV pool and (optionally) the hipGraph-captured
decode path: decode steps at a given batch size are launch-bound (dozens of
small kernels), so the runner captures one graph per padded batch-size
bucket and replays it with fresh inputs copied into static buffers
(guide: "capture launch-bound inner loops in hipGraphs").  This is the
MI355X-native replacement for the model-execution half the reference
delegates to SGLang (SURVEY §2.3 prefill/decode engine rows).
"""
from __future__ import annotations

import logging
from typing import Dict, List, Optional, Tuple

import numpy as np
import torch

from ..models.llama import PPContext, TPContext
from ..models.registry import build_model
from .batch import ForwardBatch, VarlenLayout, table_array
from .config import EngineConfig
from .sequence import Sequence

log = logging.getLogger(__name__)

GRAPH_BATCH_SIZES = (1, 2, 4, 8, 16, 24, 32, 48, 64, 96, 128, 192, 256)


class ModelRunner:
    def __init__(self, cfg: EngineConfig, tp: Optional[TPContext] = None,
                 pp: Optional[PPContext] = None):
        self.cfg = cfg
        self.device = torch.device(cfg.device)
        torch.manual_seed(cfg.seed)
        self.pp = pp or PPContext()
        self.model = build_model(cfg.model, self.device, tp, self.pp)
        self.cache = self.model.make_cache(cfg)
        self.mixed_steps = (self.model.mixed_steps if cfg.mixed_steps is None
                            else bool(cfg.mixed_steps))
        if self.mixed_steps and not self.model.mixed_steps:
            raise ValueError(f"{cfg.model.name}: mixed steps not supported")
        self.max_pages_per_seq = (cfg.max_seq_len + cfg.page_size - 1) // \
            cfg.page_size
        self._graphs: Dict[int, Tuple] = {}
        self._graph_pool = None
        # device-resident decode inputs of the last batch composition
        self._dstate: Optional[dict] = None
        log.info("model %s on %s: %d KV pages (%.1f GB pool)",
                 cfg.model.name, self.device, self.cache.num_pages,
                 self.cache.kv.numel() * self.cache.kv.element_size() / 1e9)

    # ------------------------------------------------------------------

    def _i32(self, data) -> torch.Tensor:
        return torch.tensor(data, dtype=torch.int32, device=self.device)

    def _join(self, parts: List[np.ndarray]) -> torch.Tensor:
        return torch.from_numpy(np.concatenate(parts)).to(self.device)

    # one sequence's part of a varlen step: tokens at [start, start + len)
    Chunk = Tuple[Sequence, int, List[int]]

    @torch.inference_mode()
    def run_chunks(self, chunks: List[Chunk]) -> Tuple[torch.Tensor,
                                                       List[int]]:
        """One varlen forward over portions of several sequences — a full
        prompt, a cached-prefix suffix, a piece of a long prompt or (models
        with mixed steps) a single decoded token beside them.  Returns the
        last stage's hidden rows and each chunk's first row; the rows of
        single-token chunks with a past come first."""
        order = list(range(len(chunks)))
        num_decode = 0
        if self.model.mixed_steps:
            single = [len(t) == 1 and start > 0 for _, start, t in chunks]
            num_decode = sum(single)
            order.sort(key=lambda i: not single[i])
        # numpy pieces: a step of many tokens is on the GPU's critical path
        tokens: List[np.ndarray] = []
        prev: List[np.ndarray] = []
        positions: List[np.ndarray] = []
        slots: List[np.ndarray] = []
        gather: List[np.ndarray] = []
        cu = [0]
        cu_k = [0]
        first_row = [0] * len(chunks)
        starts, ends, tables = [], [], []
        any_past = any(start > 0 for _, start, _ in chunks)
        for i in order:
            seq, start, toks = chunks[i]
            end = start + len(toks)
            tokens.append(np.asarray(toks, dtype=np.int64))
            if self.model.needs_prev:
                prev += [np.array([seq.token_at(start - 1)]), tokens[-1][:-1]]
            positions.append(np.arange(start, end, dtype=np.int32))
            slots.append(seq.block_table.slots_for(start, end - start))
            first_row[i] = cu[-1]
            cu.append(cu[-1] + (end - start))
            cu_k.append(cu_k[-1] + end)
            if any_past and not self.model.varlen:
                gather.append(seq.block_table.slots_for(0, end))
            starts.append(start)
            ends.append(end)
            tables.append(seq.block_table)
        batch = ForwardBatch(
            mode="prefill",
            positions=self._join(positions),
            slot_mapping=self._join(slots),
            cu_seqlens=self._i32(cu))
        if self.model.needs_prev:
            batch.prev_tokens = self._join(prev)
        if self.model.varlen:
            batch.starts = self._i32(starts)
            batch.state_slots = self._i32([t.state_slot for t in tables])
            batch.num_decode = num_decode
            batch.layout = VarlenLayout(starts, ends, tables, num_decode,
                                        self.cfg.page_size, self.device)
            batch.cu_prefill = self._i32([c - num_decode
                                          for c in cu[num_decode:]])
            if num_decode:
                batch.block_tables = torch.from_numpy(table_array(
                    tables[:num_decode])).to(self.device)
                batch.context_lens = self._i32(ends[:num_decode])
        elif any_past:
            batch.cu_seqlens_k = self._i32(cu_k)
            batch.kv_gather_slots = self._join(gather)
        # decode inputs that were left on the device are behind now
        self._dstate = None
        hidden_in = None
        if not self.pp.first:
            hidden_in = self.pp.recv_prev(
                (cu[-1], self.model.stream_width),
                self.model.stream_dtype, self.device)
        hidden = self.model.forward(self._join(tokens), batch, self.cache,
                                    hidden=hidden_in)
        if not self.pp.last:
            self.pp.send_next(hidden)
        return hidden, first_row

    def prefill(self, seqs: List[Sequence]) -> List[int]:
        """One prefill step: each sequence contributes its current chunk
        [num_prefilled, num_prefilled + chunk_len).  Only sequences whose
        chunk reaches the prompt end get a token sampled."""
        return self.mixed(seqs, [])

    @torch.inference_mode()
    def mixed(self, prefills: List[Sequence],
              decodes: List[Sequence]) -> List[int]:
        """One step of prompt chunks and decoded tokens as one batch."""
        chunks: List[ModelRunner.Chunk] = []
        sampled: List[Sequence] = []
        at: List[int] = []              # chunk of each sampled sequence
        for seq in decodes:
            sampled.append(seq)
            at.append(len(chunks))
            chunks.append((seq, seq.num_tokens - 1, [seq.last_token]))
        for seq in prefills:
            start = seq.num_prefilled
            end = start + (seq.chunk_len or
                           (seq.num_prompt_tokens - start))
            if end == seq.num_prompt_tokens:
                sampled.append(seq)
                at.append(len(chunks))
            chunks.append((seq, start, seq.prompt_tokens[start:end]))
            seq.num_prefilled = end
        hidden, first_row = self.run_chunks(chunks)
        if not sampled:
            return []
        if self.pp.last:
            last = [first_row[i] + len(chunks[i][2]) - 1 for i in at]
            logits = self.model.logits(hidden, self._i32(last))
            next_dev = self.sample_device(logits, sampled)[0]
        else:
            next_dev = torch.empty(len(sampled), dtype=torch.int64,
                                   device=self.device)
        if self.pp.size > 1:
            next_dev = self.pp.broadcast_tokens(next_dev)
        next_tokens = next_dev.tolist()
        for seq, tok in zip(sampled, next_tokens):
            seq.append_token(tok)
        return next_tokens

    @torch.inference_mode()
    def feed(self, chunks: List[Chunk],
             want: List[List[int]]) -> torch.Tensor:
        """Teacher-forced step: runs the given tokens as one batch, as
        generation would (single tokens alone are a decode step), and returns
        the logits at the wanted places of each chunk, in order."""
        if all(len(t) == 1 and start > 0 for _, start, t in chunks):
            self._dstate = None
            logits = self._decode_logits([seq for seq, _, _ in chunks])
            rows = [i for i, w in enumerate(want) for _ in w]
            return logits[torch.tensor(rows, dtype=torch.int64,
                                       device=self.device)]
        hidden, first_row = self.run_chunks(chunks)
        rows = [first_row[i] + p for i, w in enumerate(want) for p in w]
        return self.model.logits(hidden, self._i32(rows))

    # ------------------------------------------------------------------

    def _build_decode_state(self, seqs: List[Sequence]) -> dict:
        """Device-resident decode inputs.  Valid across steps for the same
        batch composition: positions/ctx advance on-device, the block tables
        never change mid-decode (pages are reserved for prompt+max_new at
        admission — engine/scheduler.py), so the only host->device traffic
        per step is nothing at all; sampled tokens stay on-device as the
        next step's input."""
        dev = self.device
        positions = self._i32([seq.num_tokens - 1 for seq in seqs])
        ctx = self._i32([seq.num_tokens for seq in seqs])
        tokens = torch.tensor([seq.last_token for seq in seqs],
                              dtype=torch.int64, device=dev)
        bt_np = table_array([seq.block_table for seq in seqs])
        state = {"ids": tuple(s.seq_id for s in seqs),
                 "positions": positions, "ctx": ctx, "tokens": tokens,
                 "bt": torch.from_numpy(bt_np).to(dev), "fresh": True,
                 "state_slots": None, "prev": None}
        if self.model.needs_prev:
            state["prev"] = torch.tensor(
                [seq.token_at(seq.num_tokens - 2) for seq in seqs],
                dtype=torch.int64, device=dev)
        if self.model.stateful:
            state["state_slots"] = self._i32(
                [seq.block_table.state_slot for seq in seqs])
        return state

    def _decode_slots(self, state: dict) -> torch.Tensor:
        ps = self.cfg.page_size
        pos = state["positions"].long()
        page = torch.gather(state["bt"], 1,
                            (pos // ps).unsqueeze(1)).squeeze(1)
        return (page * ps + (pos % ps).to(torch.int32)).to(torch.int32)

    def _decode_logits(self, seqs: List[Sequence]) -> Optional[torch.Tensor]:
        """Forward of one decode step; logits [n, vocab] on the last stage."""
        n = len(seqs)
        ids = tuple(s.seq_id for s in seqs)
        state = self._dstate
        if state is None or state["ids"] != ids:
            state = self._build_decode_state(seqs)
            self._dstate = state
        elif not state["fresh"]:
            state["positions"] += 1
            state["ctx"] += 1
        state["fresh"] = False
        slots = self._decode_slots(state)
        use_graph = (not self.cfg.enforce_eager and
                     self.device.type == "cuda" and
                     self.pp.size == 1 and           # p2p hops: eager path
                     self.model.tp.graph_safe and    # xGMI AR or no TP
                     n <= GRAPH_BATCH_SIZES[-1])
        if use_graph:
            return self._decode_graph(state, slots, n)[:n]
        batch = self._decode_batch(state, slots, n)
        hidden_in = None
        if not self.pp.first:
            hidden_in = self.pp.recv_prev(
                (n, self.model.stream_width),
                self.model.stream_dtype, self.device)
        hidden = self.model.forward(state["tokens"], batch, self.cache,
                                    hidden=hidden_in)
        if self.pp.last:
            return self.model.logits(hidden)
        self.pp.send_next(hidden)
        return None

    def _decode_batch(self, inputs: dict, slots: torch.Tensor,
                      n: int) -> ForwardBatch:
        return ForwardBatch(
            mode="decode", positions=inputs["positions"], slot_mapping=slots,
            block_tables=inputs["bt"], context_lens=inputs["ctx"],
            starts=inputs["positions"], state_slots=inputs["state_slots"],
            prev_tokens=inputs["prev"],
            decode_num_splits=self.model.decode_splits(
                n, self.cfg.max_seq_len))

    @torch.inference_mode()
    def decode(self, seqs: List[Sequence]) -> List[int]:
        n = len(seqs)
        logits = self._decode_logits(seqs)
        state = self._dstate
        if self.pp.last:
            next_dev, next_tokens = self.sample_device(logits, seqs)
        else:
            next_dev = torch.empty(n, dtype=torch.int64, device=self.device)
        if self.pp.size > 1:
            next_dev = self.pp.broadcast_tokens(next_dev)
            next_tokens = next_dev.tolist()
        if state["prev"] is not None:
            state["prev"] = state["tokens"]
        state["tokens"] = next_dev
        for seq, tok in zip(seqs, next_tokens):
            seq.append_token(tok)
        return next_tokens

    # ------------------------------------------------------------------

    def _graph_bucket(self, n: int) -> int:
        for b in GRAPH_BATCH_SIZES:
            if n <= b:
                return b
        return GRAPH_BATCH_SIZES[-1]

    def _build_graph(self, bs: int):
        """Capture one decode step at batch size ``bs`` into a hipGraph."""
        static = {
            "tokens": torch.zeros(bs, dtype=torch.int64, device=self.device),
            "prev": torch.zeros(bs, dtype=torch.int64, device=self.device),
            "positions": torch.zeros(bs, dtype=torch.int32, device=self.device),
            "slots": torch.zeros(bs, dtype=torch.int32, device=self.device),
            "ctx": torch.ones(bs, dtype=torch.int32, device=self.device),
            "bt": torch.zeros(bs, self.max_pages_per_seq, dtype=torch.int32,
                              device=self.device),
            # padding rows use the scratch slot 0
            "state_slots": torch.zeros(bs, dtype=torch.int32,
                                       device=self.device),
        }
        batch = self._decode_batch(static, static["slots"], bs)
        # warm up allocations outside capture
        torch.cuda.synchronize()
        hidden = self.model.forward(static["tokens"], batch, self.cache)
        logits = self.model.logits(hidden)
        torch.cuda.synchronize()
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(graph, pool=self._graph_pool):
            hidden = self.model.forward(static["tokens"], batch, self.cache)
            logits = self.model.logits(hidden)
        if self._graph_pool is None:
            self._graph_pool = graph.pool()
        self._graphs[bs] = (graph, static, logits)
        log.info("captured decode hipGraph for batch %d", bs)
        return self._graphs[bs]

    def _decode_graph(self, state: dict, slots: torch.Tensor,
                      n: int) -> torch.Tensor:
        bs = self._graph_bucket(n)
        if bs not in self._graphs:
            self._build_graph(bs)
        graph, static, logits = self._graphs[bs]
        static["tokens"][:n].copy_(state["tokens"][:n])
        static["positions"][:n].copy_(state["positions"])
        static["slots"][:n].copy_(slots)
        static["ctx"][:n].copy_(state["ctx"])
        if state["state_slots"] is not None:
            static["state_slots"][:n].copy_(state["state_slots"])
        if state["prev"] is not None:
            static["prev"][:n].copy_(state["prev"])
        bt = state["bt"]
        if state.get("graph_bt_loaded") != (state["ids"], bs):
            # block tables are stable for this batch: upload once per batch
            static["bt"].zero_()
            static["bt"][:n, :bt.shape[1]].copy_(bt)
            if n < bs:
                # padding rows decode against page 0 with ctx=1: harmless
                # work; their slot writes land in reserved scratch page 0
                static["slots"][n:] = 0
                static["positions"][n:] = 0
                static["ctx"][n:] = 1
                static["state_slots"][n:] = 0
            state["graph_bt_loaded"] = (state["ids"], bs)
        graph.replay()
        return logits

    # ------------------------------------------------------------------

    @torch.inference_mode()
    def sample(self, logits: torch.Tensor, seqs: List[Sequence]) -> List[int]:
        return self.sample_device(logits, seqs)[1]

    @torch.inference_mode()
    def sample_device(self, logits: torch.Tensor, seqs: List[Sequence]):
        """Returns (device int64 tensor, host list) of next tokens — the
        device tensor feeds the next decode step without a host round trip."""
        temps = [seq.sampling.temperature for seq in seqs]
        if all(t == 0.0 for t in temps):
            dev = logits.argmax(dim=-1)
        else:
            t = torch.tensor([max(tt, 1e-5) for tt in temps],
                             device=logits.device).unsqueeze(1)
            probs = torch.softmax(logits / t, dim=-1)
            dev = torch.multinomial(probs, 1).squeeze(1)
        return dev, dev.tolist()
