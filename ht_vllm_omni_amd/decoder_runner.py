"""DecoderModelRunner: the two-phase runner contract (execute_model / sample_tokens) over ``DecoderEngine``.

The persistent batch, block tables, hipGraph buckets, pinned uploads, asynchronous outputs and log-probabilities are
``MI355XARModelRunner``'s.  What differs: prompts are token ids, each row also owns a state slot, a step is ONE forward -- portions of
prompts beside decoded tokens -- and a prompt may stay open and be fed in pieces, with the logits of chosen places returned.

Row invariant of a step: decoded tokens first, then the prompts that complete in the step, then the rest; the rows that sample are a prefix.
A step of decoded tokens only replays the captured decode step.
"""
from __future__ import annotations

from dataclasses import dataclass, field

import numpy as np
import torch

from .payloads import EMPTY_MODEL_RUNNER_OUTPUT, LogprobsLists, OmniModelRunnerOutput, OmniSchedulerOutput, SamplingParams
from .runner import MI355XARModelRunner, _HostRecord, _Range, _ROW_BUFFERS, _StepState
from .sched import SlotPool


@dataclass
class DecoderRequestState:
    req_id: str
    prompt_ids: list[int]
    block_ids: list[int]
    sampling: SamplingParams
    open_prompt: bool = False
    num_computed: int = 0
    output_ids: list[int] = field(default_factory=list)
    n_sampled: int = 0                  # tokens sampled so far, including those of steps whose ids the host has not read
    prefill_len: int = 0                # tokens whose ids the host supplies: the prompt, after a preemption also the outputs recomputed with it

    @property
    def in_decode(self) -> bool:
        return self.num_computed >= self.prefill_len


class DecoderModelRunner(MI355XARModelRunner):
    row_buffers = tuple(n for n in _ROW_BUFFERS if n != "last_hidden") + ("state_slot",)

    def __init__(self, engine, **kw):
        super().__init__(engine, engine_output_type="text", **kw)
        self.slots = SlotPool(engine.max_batch)

    # ------------------------------------------------------------------ persistent batch
    def _reset_row(self, r: int) -> None:
        super()._reset_row(r)
        self.engine.state_slot[r] = 0

    def _left_batch(self, rid: str) -> None:
        self.slots.release(rid)

    def _fed(self, st: DecoderRequestState, token_ids: list[int]) -> None:
        st.prompt_ids.extend(token_ids)
        st.prefill_len += len(token_ids)

    def _place(self, st: DecoderRequestState, row_sampling: dict) -> None:
        """A request into the next free row with a state slot of its own."""
        e = self.engine
        self.requests[st.req_id] = st
        r = len(self.rows)
        self.rows.append(st.req_id)
        self._reset_row(r)
        e.set_row_sampling(r, **row_sampling)
        e.block_table[r, :len(st.block_ids)] = self._up(st.block_ids, torch.int32)
        e.state_slot[r] = self.slots.acquire(st.req_id)

    def _admit(self, nr) -> None:
        sp = nr.sampling_params or self.default_sampling
        row_sampling = self._row_sampling(nr.req_id, sp)
        ids = [int(t) for t in nr.prompt_token_ids or ()]
        if not ids or min(ids) < 0 or max(ids) >= self.d.vocab:
            raise ValueError(f"request {nr.req_id}: prompt_token_ids missing or outside the vocabulary")
        if not nr.open_prompt and self.d.vocab > self.engine.MAX_SAMPLED_VOCAB:
            raise ValueError(f"request {nr.req_id}: the sampler takes vocabularies of up to {self.engine.MAX_SAMPLED_VOCAB} tokens")
        self._place(DecoderRequestState(nr.req_id, ids, list(nr.block_ids[0]), sp, open_prompt=nr.open_prompt, num_computed=int(nr.num_computed_tokens),
                                        prefill_len=len(ids)), row_sampling)

    def _resume(self, rid: str, block_ids: list[int], num_computed: int, nr=None) -> None:
        """A preempted request comes back with new blocks: its cache and state are rebuilt from the prompt and everything it emitted."""
        st = self.preempted.pop(rid)
        if st.n_sampled != len(st.output_ids):
            raise RuntimeError(f"request {rid}: resumed with {st.n_sampled - len(st.output_ids)} sampled token(s) still in flight")
        if nr is not None and nr.prompt_token_ids is not None:
            st.prompt_ids = [int(t) for t in nr.prompt_token_ids]
        st.block_ids, st.num_computed, st.prefill_len = list(block_ids), int(num_computed), len(st.prompt_ids) + len(st.output_ids)
        self._place(st, self._row_sampling(rid, st.sampling))

    def _start_sampling(self, r: int, st: DecoderRequestState) -> None:
        """Row r samples its next token behind a prompt (or a recomputed sequence): counters of the sampler at that token."""
        e = self.engine
        e.positions[r] = st.prefill_len - 1
        e.seq_lens[r] = st.prefill_len
        e.steps[r] = len(st.output_ids)
        e.seen[r].zero_()
        e.seen[r, self._up(st.prompt_ids + st.output_ids, torch.long)] = 1

    # ------------------------------------------------------------------ phase 1
    @torch.inference_mode()
    def execute_model(self, scheduler_output: OmniSchedulerOutput, intermediate_tensors=None):
        so = scheduler_output
        if self.execute_model_state is not None:
            raise RuntimeError("State error: sample_tokens() must be called after execute_model() returns None.")
        if so.finished_requests_needing_kv_transfer:
            raise ValueError("language models hand no cache to another stage")
        with _Range("gpu_model_runner: preprocess"):
            self._update_states(so)
        if not so.total_num_scheduled_tokens:
            return EMPTY_MODEL_RUNNER_OUTPUT
        sched, e = so.num_scheduled_tokens, self.engine
        dec, done, part, idle = [], [], [], []
        for r, rid in enumerate(self.rows):
            n, st = sched.get(rid, 0), self.requests[rid]
            if n <= 0:
                idle.append(r)
            elif st.in_decode:
                if n != 1:
                    raise RuntimeError(f"request {rid}: decoded tokens are scheduled one per step")
                dec.append(r)
            elif st.num_computed + n > st.prefill_len:
                raise RuntimeError(f"request {rid}: scheduled past the tokens it has")
            elif st.num_computed + n == st.prefill_len and not st.open_prompt:
                done.append(r)
            else:
                part.append(r)
        self._permute_rows(dec + done + part + idle)
        nd, ns = len(dec), len(dec) + len(done)
        logits = {}
        with _Range("gpu_model_runner: forward"):
            if done or part or any(rid in so.logits_at for rid in self.rows[:nd]):
                logits = self._run_batch(so, nd, ns, ns + len(part))
            else:
                self._run_decode(nd)
        lp = {}
        k = self._wants_logprobs([self.requests[rid] for rid in self.rows[:ns]])
        if k >= 0:
            lp["rows"] = (list(range(ns)), self._logprob_rows(e.logits[:ns, :self.d.vocab], e.input_ids[:ns], k))
        rows = []
        for r, rid in enumerate(self.rows):
            n = sched.get(rid, 0)
            if n > 0:
                st = self.requests[rid]
                st.num_computed += n
                st.n_sampled += r < ns
                rows.append((r, rid, st))
        stt = _StepState(so, list(range(nd)), {}, None, {}, rows, len(self.rows), lp)
        stt.n_sampled_rows, stt.token_logits = ns, logits
        self.execute_model_state = stt
        return None

    def _run_batch(self, so: OmniSchedulerOutput, nd: int, ns: int, nrows: int) -> dict:
        """Rows [0, nrows) as one forward: decoded tokens [0, nd) by their device ids, the others by the request's tokens; rows [0, ns) sample."""
        e, sched = self.engine, so.num_scheduled_tokens
        segs = []                                                 # (row, first position, tokens or None for a device id)
        for r in range(nrows):
            st = self.requests[self.rows[r]]
            n, p = sched[st.req_id], st.num_computed
            toks = None if r < nd else (st.prompt_ids + st.output_ids)[p:p + n]
            segs.append((r, p, n, toks))
        segs.sort(key=lambda s: s[2] > 1)                         # single tokens first (stable): they take the decode attention
        ones = sum(1 for s in segs if s[2] == 1)
        ids, row, pos, first, at = [], [], [], {}, 0
        for r, p, n, toks in segs:
            ids.append(np.zeros(n, np.int32) if toks is None else np.asarray(toks, np.int32))
            row.append(np.full(n, r, np.int32))
            pos.append(np.arange(p, p + n, dtype=np.int32))
            first[r] = at
            at += n
        b = e.make_batch(np.concatenate(ids), np.concatenate(row), np.concatenate(pos), [s[2] for s in segs[ones:]], n_decode=ones,
                         max_keys=max([s[1] + 1 for s in segs[:ones]] or [0]))
        if nd:
            b.ids[:nd] = e.input_ids[:nd]                         # rows [0, nd) are the first single-token segments, in row order
        # places whose logits are needed: the sampling rows' last tokens, then what the step was asked for
        last = [first[r] + sched[self.rows[r]] - 1 for r in range(ns)]
        want, spans = [], {}
        for r in range(nrows):
            rid = self.rows[r]
            if rid in so.logits_at:
                spans[rid] = (len(want), len(so.logits_at[rid]))
                want += [first[r] + k for k in so.logits_at[rid]]
        out = e.forward(b, sel=self._up(last + want, torch.int32) if last or want else torch.empty(0, dtype=torch.int32, device=b.ids.device))
        if ns:
            e.logits[:ns] = out[:ns]
            for r in range(nd, ns):
                self._start_sampling(r, self.requests[self.rows[r]])
            e.num_live.fill_(ns)
            self._num_live = ns
            e.sample_rows_in_place(ns, e.num_live)
        return {rid: out[ns + o:ns + o + n, :self.d.vocab] for rid, (o, n) in spans.items()}

    # ------------------------------------------------------------------ phase 2
    def _collect(self, stt: _StepState, pending) -> _HostRecord:
        n = stt.n_rows
        if pending is None:
            ids = self.engine.ids_status[:n].cpu()
        else:
            _, slot, ev, _ = pending
            with torch.cuda.stream(self._copy_stream):
                self._copy_stream.wait_event(ev)
                ids = slot[:n].cpu()
        return _HostRecord(ids.tolist(), [0, 0, 0, 0], None, None, {}, logprobs=self._logprobs_host(stt))

    def _bookkeep(self, stt: _StepState, rec: _HostRecord, kv_extracted) -> OmniModelRunnerOutput:
        req_ids, sampled, lps = [], [], []
        for r, rid, st in stt.sched_rows:
            tok = [int(rec.ids[r])] if r < stt.n_sampled_rows else []
            st.output_ids += tok
            req_ids.append(rid)
            sampled.append(tok)
            lps.append(rec.logprobs.get(r) if tok else None)
        want = bool(rec.logprobs)
        return OmniModelRunnerOutput(
            req_ids=req_ids, req_id_to_index={rid: i for i, rid in enumerate(req_ids)}, sampled_token_ids=sampled,
            logprobs=LogprobsLists([t[0] if t else [] for t in lps], [t[1] if t else [] for t in lps], [t[2] if t else 0 for t in lps]) if want else None,
            num_nans_in_logits={rid: t[3] for rid, t in zip(req_ids, lps) if t} if want else None,
            cudagraph_stats=dict(self.cudagraph_stats), token_logits=stt.token_logits or None)
