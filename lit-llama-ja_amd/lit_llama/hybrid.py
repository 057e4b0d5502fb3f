"""What the models with per-sequence state (state.SequenceState) share: reading of their config objects, scratch of
a forward call, and the calls around `run` -- packed rows in, logits out.

A model provides `config`, `mixers`, `dtype`, `device`, `head` (its output PackedLinear), `new_work(M, head_rows)`
and `run(rows, work, state, logits, pick, stream, taps)`.
"""
from __future__ import annotations

from typing import Optional

import torch

from . import _hip
from .state import Rows, SequenceState

MAX_POSITIONS = 1 << 30  # positions are int32; the layers themselves have no length limit


def take_values(d: dict, where: str, **kinds) -> list:
    """Values of a config object with exactly these keys; a kind with a default (kind, default) is optional."""
    if not isinstance(d, dict):
        raise ValueError(f"config: {where} is not an object")
    extra = set(d) - set(kinds)
    if extra:
        raise ValueError(f"config: {where} has unknown keys {sorted(extra)}")
    out = []
    for key, kind in kinds.items():
        default = ()
        if isinstance(kind, tuple):
            kind, default = kind[0], kind[1:]
        if key not in d:
            if not default:
                raise ValueError(f"config: {where} has no '{key}'")
            out.append(default[0])
            continue
        v = d[key]
        if v is None and default == (None,):
            out.append(None)
            continue
        if kind is int and (isinstance(v, bool) or int(v) != v):
            raise ValueError(f"config: {where}.{key} is not an integer")
        out.append(kind(v) if kind in (int, float) else v)
    return out


class Scratch:
    """Scratch of a forward call over M rows (a decode session keeps one for all its steps)."""

    def __init__(self, M: int, device):
        self.device = device
        self.all_rows = torch.arange(M, dtype=torch.int32, device=device)
        self.hb = None  # the head's input rows
        self._buffers: dict = {}

    def head_rows(self, n: int, width: int, dtype) -> torch.Tensor:
        if self.hb is None or self.hb.shape[0] < n:
            self.hb = torch.empty(n, width, dtype=dtype, device=self.device)
        return self.hb

    def buffer(self, name: str, numel: int, dtype, zero: bool = False) -> torch.Tensor:
        """Scratch shared by the layers, at least numel long; zero: cleared when it is made."""
        t = self._buffers.get(name)
        if t is None or t.numel() < numel:
            t = self._buffers[name] = (torch.zeros if zero else torch.empty)(numel, dtype=dtype, device=self.device)
        return t


class TensorReader:
    """Takes a checkpoint's tensors by name, with their shapes checked; what is left over is an error."""

    def __init__(self, tensors: dict):
        self.left = dict(tensors)

    def take(self, name: str, shape) -> torch.Tensor:
        if name not in self.left:
            raise ValueError(f"tensor {name} is missing")
        t = self.left.pop(name)
        if tuple(t.shape) != tuple(shape):
            raise ValueError(f"tensor {name} has shape {tuple(t.shape)}, expected {tuple(shape)}")
        return t

    def group(self, prefix: str) -> dict:
        return {k[len(prefix):]: self.left.pop(k) for k in [n for n in self.left if n.startswith(prefix)]}

    def done(self) -> None:
        if self.left:
            raise ValueError(f"unexpected tensors {sorted(self.left)}")


class HybridModel(torch.nn.Module):
    def session_program(self, sess):
        from .engine import HybridProgram

        return HybridProgram(sess)

    def act_dtype(self) -> torch.dtype:
        return self.dtype

    def new_state(self, slots: int, max_length: Optional[int] = None) -> SequenceState:
        return SequenceState(self, slots, max_length)

    def check_tokens(self, tokens) -> None:
        if len(tokens) and not 0 <= min(tokens) <= max(tokens) < self.config.vocab_size:
            raise ValueError(f"token ids must be in [0, {self.config.vocab_size})")

    @torch.no_grad()
    def extend(self, state: SequenceState, slots: list, starts: list, tokens: list, want: Optional[list] = None,
               taps: Optional[list] = None) -> torch.Tensor:
        """Run each sequence's next tokens (lists of ids) from its state. Returns the logits (n, vocab) at
        the wanted places, want[b] a list of indices into tokens[b] (None: all), in that order."""
        for t in tokens:
            self.check_tokens(t)
        rows = Rows.packed(tokens, starts, slots, self.device)
        if want is None:
            pick, n = None, rows.M
        else:
            base, idx = 0, []
            for t, ks in zip(tokens, want):
                if ks and not 0 <= min(ks) <= max(ks) < len(t):
                    raise ValueError("wanted places must be among the tokens given")
                idx += [base + k for k in ks]
                base += len(t)
            pick, n = torch.tensor(idx, dtype=torch.int32).to(self.device), len(idx)
        state.ensure(max(s + len(t) for s, t in zip(starts, tokens)))
        logits = torch.empty(n, self.head.Np, dtype=self.dtype, device=self.device)
        self.run(rows, self.new_work(rows.M), state, logits, pick, _hip.stream(), taps)
        return logits[:, :self.config.vocab_size]

    @torch.no_grad()
    def forward(self, idx: torch.Tensor, max_seq_length: Optional[int] = None,
                input_pos: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Logits (B, T, vocab) of B equal-length sequences, as LLaMA.forward: without input_pos from their
        first token on a state of their own; with it (contiguous positions) going on from the model's
        kept state, which the call with position 0 begins (reset_cache() ends it)."""
        B, T = idx.shape
        toks = idx.tolist()
        if input_pos is None:
            state = self.new_state(B, T)
            return self.extend(state, state.alloc(B), [0] * B, toks).view(B, T, -1)
        p = input_pos.tolist()
        if p != list(range(p[0], p[0] + T)):
            raise ValueError("input_pos must be T contiguous positions")
        if getattr(self, "_kept", None) is None:
            if p[0] != 0:
                raise ValueError("the first call with input_pos must begin at position 0")
            self._kept = (state := self.new_state(B, max_seq_length), state.alloc(B), [0] * B)
        state, slots, seen = self._kept
        if len(slots) != B or seen[0] != p[0]:
            raise ValueError(f"expected {len(slots)} sequences at position {seen[0]}; call reset_cache() first")
        out = self.extend(state, slots, seen, toks).view(B, T, -1)
        self._kept = (state, slots, [p[0] + T] * B)
        return out

    def reset_cache(self) -> None:
        self._kept = None
