"""Decode session: the reference's token loop (generate.py:61-87) with the per-token work
captured once into a HIP graph.

One decode step = embedding of the current token (which also advances the device-side
position), the n_layer fused blocks, ln_f + lm_head and the next-token choice -- the greedy
argmax (top_k = 1) or the temperature / top-k sampler (llj_sample, generate.py:66-74; its
uniform comes from a counter hash of (seed, position, row), or from a caller's table of
uniforms per position) -- which writes the next token both into `cur` and into the output id
buffer. Nothing in the step reads the host, so replaying the graph K times generates K tokens
with no host round trip (the reference syncs per layer at model.py:221 and per token at
generate.py:86).

Batch B > 1 decodes B equal-length prompts together (each row equals an independent B=1
run: tests/test_model_gpu.py); the reference's generate() is batch 1 only (generate.py:62). Up to 8
rows share every fused launch; larger batches take the ops in row slices.

The model-specific half of a session is its program (model.session_program(session)): what a prompt
call and a decode step launch, and what they keep. LLaMAProgram drives the K / V cache models (one
position shared by the rows); HybridProgram drives models with per-sequence state (state.SequenceState:
recurrent states, latent rings and K / V rows behind a slot per sequence), whose prompts may differ in length and
whose sequences may end one by one (`finish`). `feed` runs a step on given tokens instead of the chosen
ones.
"""
from __future__ import annotations

import torch

from . import _hip
from .model import LLaMA, _Work, _enable_i8_handoff
from .state import Rows


class LLaMAProgram:
    """Prompt and step launches of LLaMA.forward's blocks over the ring K / V caches; one position for all rows."""

    npos = 1

    def __init__(self, sess: "DecodeSession"):
        self.sess = sess
        self.dev = sess.model.transformer.wte.weight.device
        _hip.require_device(sess.model.transformer.wte.weight, "model")

    def prefill(self, prompts: torch.Tensor) -> int:
        s = self.sess
        m = s.model
        if not isinstance(prompts, torch.Tensor) or prompts.dim() != 2:
            raise ValueError("this model decodes equal-length prompts: pass a (B, T) tensor")
        B, T = prompts.shape
        assert B == s.B and T + 1 <= s.total
        m.reset_cache()
        m.kv_caches = m._alloc_kv(B, s.S, self.dev)
        if m.rope_cache is None:
            m.rope_cache = m.build_rope_cache(prompts)
        pos = torch.arange(T, device=self.dev, dtype=torch.int32)
        m._run(prompts.to(self.dev), pos, s.S, m.kv_caches, last_only_out=s.logits)
        s.tokens[:, :T] = prompts.to(torch.int32)
        s.pos.fill_(T - 1)
        return T

    def prepare(self) -> None:
        """decode-step operands (fixed for the session)"""
        s = self.sess
        m = s.model
        s.specs = m._layer_specs()
        if m._generic():  # the any-shape kernels (csrc/generic.hip)
            s.work = _Work(m.config, s.B, self.dev, False, s.S, generic=True, dtype=m.act_dtype())
        else:
            need_i8 = any(q[0] == 2 for layer in s.specs["layers"] for q in layer) or s.specs["head"][0] == 2
            s.work = _Work(m.config, s.B, self.dev, need_i8, s.S)
            _enable_i8_handoff(s.work, s.specs)

    def reset_handoff(self):
        """The LLM.int8 hand-off blocks (_Work.y_st / h_st) must be zero when a step starts; a
        completed step leaves them so, a step that raised part-way may not: zero them again."""
        w = self.sess.work
        if w is not None and getattr(w, "y_st", None) is not None:
            w.y_st.zero_()
            w.h_st.zero_()

    def step(self, st) -> None:
        s = self.sess
        m, w, B = s.model, s.work, s.B
        cfg = m.config
        try:
            if w.generic:
                _hip.call("llj_g_embedding", s.cur.data_ptr(), m.transformer.wte.weight.data_ptr(), w.x.data_ptr(), B,
                          cfg.n_embd, s.pos.data_ptr(), w.dt, st)
            else:
                _hip.call("llj_embedding", s.cur.data_ptr(), m.transformer.wte.weight.data_ptr(), w.x.data_ptr(), B,
                          cfg.n_embd, s.pos.data_ptr(), st)
            m._blocks(w, s.specs, m.kv_caches, s.pos, B, 1, s.S, st)
            m._head(w.x, B, s.specs, s.logits, st, w)
        except BaseException:
            self.reset_handoff()
            raise

    def finish(self, live: list) -> None:
        raise NotImplementedError("rows of this model share one position: the batch ends together")


class HybridProgram:
    """Prompt and step launches of a model with per-sequence state (run / new_state); a position per row."""

    def __init__(self, sess: "DecodeSession"):
        self.sess = sess
        self.npos = sess.B
        self.dev = sess.model.device
        self.state = sess.state if sess.state is not None else sess.model.new_state(sess.B, sess.S)
        self.slots: list = []

    def prefill(self, prompts, want=None):
        """Every sequence from its first token; session.logits = the last rows' (and with `want` returns the
        logits at those places, per sequence a list of indices)."""
        s = self.sess
        m = s.model
        toks = [p.tolist() if isinstance(p, torch.Tensor) else list(p) for p in prompts]
        if len(toks) != s.B:
            raise ValueError(f"{len(toks)} prompts for a session of {s.B}")
        lens = [len(t) for t in toks]
        if s.S is not None and max(lens) > s.S:
            raise ValueError(f"prompt of {max(lens)} tokens, max_seq_length {s.S}")
        assert s.total is None or max(lens) + 1 <= s.total
        if self.slots:
            self.state.release(self.slots)
            self.slots = []
        self.state.reserve(s.B)
        self.slots = self.state.alloc(s.B)
        places = [sorted({*(want[b] if want else ()), n - 1}) for b, n in enumerate(lens)]
        out = m.extend(self.state, self.slots, [0] * s.B, toks, places)
        base, last, picked = 0, [], []
        for b, pl in enumerate(places):
            last.append(base + len(pl) - 1)
            picked += [base + pl.index(k) for k in (want[b] if want else ())]
            base += len(pl)
        s.logits[:, :out.shape[1]] = out[last]
        if s.tokens is not None:
            for b, t in enumerate(toks):
                s.tokens[b, :lens[b]] = torch.tensor(t, dtype=torch.int32)
        s.pos.copy_(torch.tensor(lens, dtype=torch.int32) - 1)
        self.seen = list(lens)  # tokens each live row's state has taken in
        self.wanted = out[picked] if want else None
        return lens

    def prepare(self) -> None:
        s = self.sess
        s.work = s.model.new_work(s.B, head_rows=s.B)
        self.slot = torch.tensor(self.slots, dtype=torch.int32).to(self.dev)

    def step(self, st) -> None:
        s = self.sess
        rows = Rows(s.B, s.B, s.cur, s.pos, self.slot)
        s.model.run(rows, s.work, self.state, s.logits, None, st)

    def room(self, n: int) -> None:
        """State for n more tokens per row."""
        if self.state.ensure(max(self.seen) + n):
            self.sess.graph = None

    def finish(self, live: list) -> None:
        kept = set(live)
        self.state.release([x for b, x in enumerate(self.slots) if b not in kept])
        self.slots, self.seen = [self.slots[b] for b in live], [self.seen[b] for b in live]

    def extend(self, live: list, tokens: list, want) -> torch.Tensor:
        """These live rows take in their next tokens (one prompt-style call); the wanted places' logits."""
        s = self.sess
        self.room(max(map(len, tokens)))
        out = s.model.extend(self.state, [self.slots[b] for b in live], [self.seen[b] for b in live], tokens, want)
        for b, t in zip(live, tokens):
            self.seen[b] += len(t)
        s.pos.copy_(torch.tensor(self.seen, dtype=torch.int32) - 1)
        return out


class DecodeSession:
    def __init__(self, model: LLaMA, batch: int, max_seq_length: int, total_len: int, use_graph: bool = True,
                 temperature: float = 1.0, top_k: int | None = 1, seed: int = 0,
                 uniforms: torch.Tensor | None = None, state=None, keep_tokens: bool = True):
        """top_k == 1: greedy; otherwise sampling at `temperature` over the top_k logits (None:
        all). uniforms: optional (total_len, batch) fp32 device table, row p = the uniforms of the
        token at position p (tests replay a reference run's draws). state: a SequenceState to
        take the sequences' slots from (models with per-sequence state; default: one of its own).
        keep_tokens False: no output id buffer (total_len, max_seq_length may be None where the model has no limit)."""
        cfg = model.config
        assert max_seq_length is None or max_seq_length <= cfg.block_size
        self.model, self.B, self.S, self.total, self.state = model, batch, max_seq_length, total_len, state
        if batch < 1:
            raise ValueError(f"decode batch {batch} < 1")
        self.program = model.session_program(self)
        self.ragged = isinstance(self.program, HybridProgram)  # a position per row, sequences of any lengths
        dev = self.program.dev
        self.dev = dev
        # batches past QKV_ROWS (8) run every fused op in row slices of 8 (16 for the plain linears)
        self.cur = torch.zeros(batch, dtype=torch.int32, device=dev)
        self.pos = torch.zeros(self.program.npos, dtype=torch.int32, device=dev)
        self.tokens = torch.zeros(batch, total_len, dtype=torch.int32, device=dev) if keep_tokens else None
        self.logits = torch.empty(batch, cfg.padded_vocab_size, dtype=model.act_dtype(), device=dev)
        # columns the next token is chosen from: LLaMA's padded rows are part of its vocabulary (the
        # reference samples over them), a table padded to the kernels' tiles only is not
        self.vocab = cfg.vocab_size if self.ragged else cfg.padded_vocab_size
        self.use_graph = use_graph
        self.graph = None
        self.t_prompt = 0
        self.steps_done = 0
        self.specs = None
        self.work = None
        self.temperature = float(temperature)
        self.top_k = 0 if top_k is None else int(top_k)
        self.seed = int(seed) & ((1 << 64) - 1)
        if uniforms is not None:
            assert uniforms.dtype == torch.float32 and uniforms.shape == (total_len, batch) and uniforms.is_contiguous()
            _hip.require_device(uniforms, "uniforms")
        self.uniforms = uniforms

    def _choose(self, st):
        """next token of every row from self.logits -> cur and tokens[:, pos + 1]"""
        _hip.call("llj_next_token", self.logits.data_ptr(), self.logits.stride(0), self.B, self.vocab, self.temperature,
                  self.top_k, _hip.ptr(self.uniforms), self.seed, self.cur.data_ptr(), _hip.ptr(self.tokens),
                  self.total or 0, self.pos.data_ptr(), 1 if self.ragged else 0,
                  1 if self.logits.dtype == torch.float32 else 0, st)

    # -- prefill: eager; fills the caches, picks the first new token
    @torch.no_grad()
    def prefill(self, prompts, want=None):
        """prompts: (B, T) ids, or for models with a position per row a list of B sequences. `want` (such
        models): also return the logits at those places of each prompt, (n, vocab)."""
        if want is None:
            lens = self.program.prefill(prompts)
        elif self.ragged:
            lens = self.program.prefill(prompts, want)
        else:
            raise ValueError("this model's sessions return the last position's logits only")
        self._choose(_hip.stream())
        self.lens = lens if self.ragged else [lens] * self.B
        self.t_prompt = max(self.lens)
        self.steps_done = 1
        self.graph = None  # the caches / operands may have changed
        self.program.prepare()
        return self.program.wanted if want is not None else None

    def _step(self):
        st = _hip.stream()
        self.program.step(st)
        self._choose(st)

    def capture(self):
        if self.graph is not None or not self.use_graph:
            return
        g = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g):
            self._step()
        self.graph = g

    @torch.no_grad()
    def decode(self, n: int) -> None:
        """Generate n more tokens per row (positions t_prompt + steps_done ...)."""
        assert self.total is None or self.t_prompt + self.steps_done + n <= self.total, "beyond the output buffer"
        limit = self.S if self.ragged and self.S is not None else self.model.config.block_size
        assert self.t_prompt + self.steps_done + n - 1 <= limit, "beyond block_size"
        if self.ragged:
            self.program.room(n)
        if self.use_graph:
            self.capture()
            for _ in range(n):
                self.graph.replay()
        else:
            for _ in range(n):
                self._step()
        self.steps_done += n
        if self.ragged:
            self.program.seen = [k + n for k in self.program.seen]

    @torch.no_grad()
    def feed(self, tokens) -> torch.Tensor:
        """One step on the given next token of every live row instead of the chosen one; its logits (B, vocab)."""
        ids = [int(t) for t in tokens]
        if len(ids) != self.B or not 0 <= min(ids) <= max(ids) < self.model.config.vocab_size:
            raise ValueError(f"feed takes one token id per live row ({self.B})")
        self.cur.copy_(torch.tensor(ids, dtype=torch.int32))
        if self.tokens is not None:
            pos = self.pos.long() + 1
            self.tokens[torch.arange(self.B, device=self.dev), pos.expand(self.B)] = self.cur
        self.decode(1)
        return self.logits[:, :self.vocab]

    def extend(self, rows, tokens, want=None) -> torch.Tensor:
        """Live rows take in several given tokens each (models with per-sequence state); logits at the wanted places."""
        if not self.ragged:
            raise NotImplementedError("this model's sessions take one token per row and step")
        return self.program.extend(list(rows), tokens, want)

    @torch.no_grad()
    def finish(self, rows) -> None:
        """End these rows (indices into the live rows): their state is given back, the others move up."""
        rows = set(rows)
        if not rows <= set(range(self.B)):
            raise ValueError(f"rows {sorted(rows)} of {self.B}")
        live = [b for b in range(self.B) if b not in rows]
        self.program.finish(live)
        idx = torch.tensor(live, dtype=torch.long, device=self.dev)
        self.cur, self.pos, self.logits = self.cur[idx], self.pos[idx], self.logits[idx]
        if self.tokens is not None:
            self.tokens = self.tokens[idx]
        self.lens = [self.lens[b] for b in live]
        self.B, self.graph = len(live), None
        if live:
            self.program.prepare()

    def output(self):
        """Token ids so far: (B, n), or a list of B rows when the prompts differ in length."""
        if len(set(self.lens)) > 1:
            return [self.tokens[b, :n + self.steps_done] for b, n in enumerate(self.lens)]
        return self.tokens[:, :self.lens[0] + self.steps_done]
