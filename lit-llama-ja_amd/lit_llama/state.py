"""Per-sequence state of models whose layers keep something other than a plain K / V cache.

`SequenceState` owns, for `slots` sequences at a time,
  * every recurrent layer's state (fp32, mixer.state_shape),
  * every latent-attention layer's ring of the last tokens' latents, one per layer that projects its own
    (layers that read another layer's latents have none), sized by the widest window among its readers,
  * every full-attention layer's K / V rows, the same buffers with a row for every position: as many as the
    longest sequence allowed, or without a limit as many as the longest has needed so far (`ensure`),
  * the previous token of each sequence (models whose embedding looks back one token).
A sequence holds a slot from `alloc` to `release`; kernels address everything through the slot number, so
the rows of a batch need not be neighbours in memory and a batch can shrink without moving state.
"""
from __future__ import annotations

import torch

ALL_POSITIONS = -1  # mixer.ring_window() of layers that keep every token
GROW_ROWS = 256  # unlimited layers grow by multiples of this many rows


class SequenceState:
    def __init__(self, model, slots: int, max_length: int | None = None):
        """max_length: no sequence will be longer (rings are capped at it); None: unbounded."""
        self.model, self.max_length = model, max_length
        self.slots = 0
        self.recurrent: dict = {}
        self.ring: dict = {}
        self.ring_rows: dict = {}
        for i, mixer in enumerate(model.mixers):
            w = mixer.ring_window()
            if w == ALL_POSITIONS:
                self.ring_rows[i] = 0 if max_length is None else max(1, max_length)
            elif w is not None:
                self.ring_rows[i] = w if max_length is None else max(1, min(w, max_length))
        self._all = [i for i, mixer in enumerate(model.mixers) if mixer.ring_window() == ALL_POSITIONS]
        self._free: list = []
        self._grow(slots)

    def _grow(self, slots: int) -> None:
        m, dev = self.model, self.model.device
        for i, mixer in enumerate(m.mixers):
            shape = mixer.state_shape()
            if shape is not None:
                self.recurrent[i] = torch.zeros(slots, *shape, dtype=torch.float32, device=dev)
            if i in self.ring_rows:
                self.ring[i] = torch.zeros(slots, self.ring_rows[i], mixer.cache_width(m.dtype), dtype=m.dtype, device=dev)
        self.prev = torch.full((slots,), -1, dtype=torch.int32, device=dev)
        self._free = list(range(slots))
        self.slots = slots

    def ensure(self, length: int) -> bool:
        """Room for sequences of `length` tokens in the layers that keep every token; True if they moved (a captured
        step must be captured again)."""
        if not self._all or length <= self.ring_rows[self._all[0]]:
            return False
        if self.max_length is not None:
            raise ValueError(f"sequence of {length} tokens in a state for {self.max_length}")
        rows = max(-(-length // GROW_ROWS) * GROW_ROWS, 2 * self.ring_rows[self._all[0]])
        for i in self._all:
            old = self.ring[i]
            new = torch.zeros(old.shape[0], rows, old.shape[2], dtype=old.dtype, device=old.device)
            new[:, :old.shape[1]] = old
            self.ring[i], self.ring_rows[i] = new, rows
        return True

    def reserve(self, n: int) -> None:
        """Room for n more sequences; only an idle state can grow."""
        if n <= len(self._free):
            return
        if len(self._free) != self.slots:
            raise RuntimeError(f"{n} sequences asked for, {len(self._free)} of {self.slots} slots free")
        self._grow(n)

    def alloc(self, n: int) -> list:
        """n slots with the state of an empty sequence."""
        if n > len(self._free):
            raise RuntimeError(f"{n} sequences asked for, {len(self._free)} of {self.slots} slots free")
        out, self._free = self._free[:n], self._free[n:]
        idx = torch.tensor(out, dtype=torch.long, device=self.prev.device)
        for s in self.recurrent.values():
            s.index_fill_(0, idx, 0.0)
        self.prev.index_fill_(0, idx, -1)  # ring rows are only read at positions the sequence has written
        return out

    def release(self, slots) -> None:
        for s in slots:
            if s in self._free or not 0 <= s < self.slots:
                raise ValueError(f"slot {s} is not in use")
        self._free.extend(slots)  # a freed slot is used again after every other free one

    def nbytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in [*self.recurrent.values(), *self.ring.values(), self.prev])


class Rows:
    """The activation rows of one forward call. `decode`: one row per sequence, positions and tokens on
    the device (`pos` is advanced by the embedding). Otherwise the packed rows of every sequence's new
    tokens, sequence b's at row0[b] .. row0[b + 1] - 1 with positions start[b] ..."""

    def __init__(self, M, B, tok, pos, slot, row_seq=None, row0=None, lengths=None, starts=None):
        self.M, self.B = M, B
        self.tok, self.pos, self.slot, self.row_seq, self.row0 = tok, pos, slot, row_seq, row0
        self.lengths, self.starts = lengths, starts
        self.decode = row_seq is None
        self.slots = None  # host copy of slot (packed rows)
        self._tables: dict = {}

    @classmethod
    def packed(cls, tokens: list, starts: list, slots: list, device) -> "Rows":
        """tokens: per sequence a list of ids."""
        lengths = [len(t) for t in tokens]
        if not lengths or min(lengths) < 1:
            raise ValueError("every sequence of a call needs at least one token")
        B, M = len(lengths), sum(lengths)
        row0 = [0]
        for n in lengths:
            row0.append(row0[-1] + n)
        meta = [t for seq in tokens for t in seq]
        meta += [s + j for s, n in zip(starts, lengths) for j in range(n)]
        meta += [b for b, n in enumerate(lengths) for _ in range(n)]
        meta += row0 + list(slots)
        d = torch.tensor(meta, dtype=torch.int32).to(device)
        r = cls(M, B, d[:M], d[M:2 * M], d[3 * M + B + 1:], d[2 * M:3 * M], d[3 * M:3 * M + B + 1], lengths, list(starts))
        r.slots = list(slots)
        return r

    def _table(self, key, make):
        if key not in self._tables:
            self._tables[key] = make()
        return self._tables[key]

    def _device(self, values: list) -> torch.Tensor:
        return torch.tensor(values, dtype=torch.int32).to(self.pos.device)

    def chunks(self, C: int):
        """Packed rows cut into chunks of at most C tokens of one sequence: (number, table [(first row, rows,
        sequence)], each sequence's first chunk), the tables on the device."""

        def make():
            tab, first, row = [], [0], 0
            for b, n in enumerate(self.lengths):
                for j in range(0, n, C):
                    tab += [row + j, min(C, n - j), b]
                row += n
                first.append(len(tab) // 3)
            d = self._device(tab + first)
            return len(tab) // 3, d[:len(tab)], d[len(tab):]

        return self._table(("chunks", C), make)

    def pairs(self, C: int):
        """Work items of causal attention over blocks of at most C rows of one sequence: (number, table [(first row,
        rows, sequence) twice]) -- a late block, which sees many keys, with an early one (rows 0: none)."""

        def make():
            tab, row = [], 0
            for b, n in enumerate(self.lengths):
                blocks = [[row + j, min(C, n - j), b] for j in range(0, n, C)]
                row += n
                while blocks:
                    late = blocks.pop()
                    tab.append(late + (blocks.pop(0) if blocks else [0, 0, 0]))
            # the items with the most keys first
            pos = [s - r0 for s, r0 in zip(self.starts, self._row0())]
            tab.sort(key=lambda w: -(pos[w[2]] + w[0] + w[1]))
            return len(tab), self._device([x for w in tab for x in w])

        return self._table(("pairs", C), make)

    def _row0(self) -> list:
        out, row = [], 0
        for n in self.lengths:
            out.append(row)
            row += n
        return out

    def keys(self, window: int):
        """The keys the packed rows of a call may see through `window`: (number, gather or None, key0, kpos0,
        nkey), per sequence the first key row, its position and the number of rows. Without earlier tokens
        the key rows are the activation rows; otherwise gather = (source rows, -1 - nothing: from the ring;
        positions; slots) of every key row."""

        def make():
            old = [min(s, window - 1) for s in self.starts]
            key0, n = [], 0
            for o, t in zip(old, self.lengths):
                key0.append(n)
                n += o + t
            kpos0 = [s - o for s, o in zip(self.starts, old)]
            nkey = [o + t for o, t in zip(old, self.lengths)]
            B = self.B
            if not any(old):
                d = self._device(key0 + kpos0 + nkey)
                return n, None, d[:B], d[B:2 * B], d[2 * B:]
            src, kpos, kslot, row = [], [], [], 0
            for b, (o, t) in enumerate(zip(old, self.lengths)):
                src += [-1] * o + list(range(row, row + t))
                kpos += range(kpos0[b], kpos0[b] + o + t)
                kslot += [self.slots[b]] * (o + t)
                row += t
            d = self._device(key0 + kpos0 + nkey + src + kpos + kslot)
            g = d[3 * B:]
            return n, (g[:n], g[n:2 * n], g[2 * n:]), d[:B], d[B:2 * B], d[2 * B:3 * B]

        return self._table(("keys", window), make)
