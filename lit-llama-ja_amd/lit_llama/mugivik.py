"""Mugivik: a decoder of gated-linear-attention and sliding-window latent-attention layers in any order,
squared-relu feed-forwards, RMS norms on the sublayers' outputs, a bigram table beside the token
embedding and a tied head.

  x = norm(embed[token] + bigram[(previous token, token)])
  per layer: x += norm1(mixer(x)); x += norm2(feed-forward(x))        (norm: x / rms(x) * (1 + w))
  logits = embed . norm(x)

The residual x is fp32. A forward call takes packed activation rows (state.Rows): the new tokens of any
number of sequences, each going on from its own state, or one decode row per sequence. Everything runs on
the library's kernels: packed projections (mixers.PackedLinear), csrc/gla.hip, csrc/latent.hip and
csrc/postnorm.hip.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple

import torch

from . import _hip
from .hybrid import MAX_POSITIONS, HybridModel, Scratch, TensorReader, take_values
from .mixers import (GatedLinearAttention, GLASpec, LatentAttention, LatentSpec, PackedLinear, ReluSquaredMLP, _dt,
                     lane_pad)
from .registry import register
from .state import Rows, SequenceState
from .utils import find_multiple


@dataclass(frozen=True)
class MugivikLayer:
    mixer: object  # GLASpec or LatentSpec
    ff: Optional[int]  # None: no feed-forward


@dataclass(frozen=True)
class MugivikConfig:
    vocab_size: int
    n_embd: int
    eps: float
    buckets: int
    mul_prev: int
    mul_cur: int
    layers: Tuple[MugivikLayer, ...]

    block_size = MAX_POSITIONS

    @property
    def padded_vocab_size(self) -> int:
        return find_multiple(self.vocab_size, 128)

    @property
    def n_layer(self) -> int:
        return len(self.layers)

    @classmethod
    def from_dict(cls, d: dict) -> "MugivikConfig":
        _, emb, layers, norm, vocab, width = take_values(d, "config.json", architecture=str, embedding=dict, layers=list,
                                                         norm=dict, vocab=int, width=int)
        (big,) = take_values(emb, "embedding", bigram=dict)
        buckets, mc, mp = take_values(big, "embedding.bigram", buckets=int, mul_cur=int, mul_prev=int)
        (eps,) = take_values(norm, "norm", eps=float)
        out = []
        for i, layer in enumerate(layers):
            where = f"layers[{i}]"
            mix, mlp, kind = take_values(layer, where, mixer=dict, mlp=(dict, None), type=str)
            if kind == "gla":
                spec = GLASpec(*take_values(mix, where + ".mixer", heads=int, dim=int, vdim=int, tau=float))
            elif kind == "latent_attention":
                heads, dim, rd, vdim, rank, mask, scale, rot, src = take_values(
                    mix, where + ".mixer", heads=int, dim=int, rot_dim=int, vdim=int, kv_rank=int, mask=dict, scale=float,
                    rot=dict, kv_from=(int, None))
                (window,) = take_values(mask, where + ".mixer.mask", size=int)
                base, dims = take_values(rot, where + ".mixer.rot", base=float, dims=int)
                if dims != rd:
                    raise ValueError(f"config: {where} rotates {dims} of rot_dim {rd} dimensions")
                if src is not None and not 0 <= src < i:
                    raise ValueError(f"config: {where}.mixer.kv_from {src} is not an earlier layer")
                spec = LatentSpec(heads, dim, rd, vdim, rank, window, scale, base, src)
                if rd % 2 or window < 1:
                    raise ValueError(f"config: {where} has an odd rot_dim or an empty window")
            else:
                raise ValueError(f"config: {where} has unknown type {kind!r}")
            ff = None
            if mlp is not None:
                ff, mk = take_values(mlp, where + ".mlp", ff=int, kind=str)
                if mk != "dense":
                    raise ValueError(f"config: {where}.mlp has unknown kind {mk!r}")
            out.append(MugivikLayer(spec, ff))
        if not out or min(vocab, width, buckets) < 1:
            raise ValueError("config: needs at least one layer, a vocabulary, a width and bigram buckets")
        return cls(vocab, width, eps, buckets, mp, mc, tuple(out))


class _Work(Scratch):
    def __init__(self, m: "Mugivik", M: int):
        dev, dt, C = m.device, m.dtype, m.Cp
        super().__init__(M, dev)
        self.x = torch.empty(M, C, dtype=torch.float32, device=dev)
        # the sublayers' input: the residual itself in float32, its bf16 copy otherwise
        self.xb = self.x if dt == torch.float32 else torch.empty(M, C, dtype=dt, device=dev)
        if dt == torch.float32 and C != m.config.n_embd:
            self.x.zero_()  # padding columns
        self.t = torch.empty(M, C, dtype=dt, device=dev)
        self.proj = torch.empty(M, max(mx.inp.Np for mx in m.mixers), dtype=dt, device=dev)
        ff = [f.up.Np for f in m.mlps if f is not None]
        self.h = torch.empty(M, max(ff), dtype=dt, device=dev) if ff else None
        # mixer outputs by width: padding columns stay zero
        self.y = {n: torch.zeros(M, lane_pad(n, dt), dtype=dt, device=dev) for n in {mx.out_width() for mx in m.mixers}}
        self.cur: dict = {}  # this call's latents by layer (prompt rows)
        self.x2 = torch.empty_like(self.x) if M == 1 else None  # the residual's other place (fused post-norm products)


@register("Mugivik")
class Mugivik(HybridModel):
    HIP_SOURCES = ("postnorm", "post_gemv", "gemm_bf16", "gla", "latent", "latent_prefill", "latent_decode", "generic",
                   "ops", "options")

    def __init__(self, config: MugivikConfig):
        super().__init__()
        self.config = config
        C, eps = config.n_embd, config.eps
        self.mixers, self.mlps = [], []
        for layer in config.layers:
            s = layer.mixer
            self.mixers.append(GatedLinearAttention(s, C, eps) if isinstance(s, GLASpec) else LatentAttention(s, C, eps))
            self.mlps.append(None if layer.ff is None else ReluSquaredMLP(layer.ff, C))
        for i, mx in enumerate(self.mixers):
            src = getattr(mx.spec, "kv_from", None)
            if src is not None:
                if not isinstance(self.mixers[src], LatentAttention):
                    raise ValueError(f"layer {i} shares the latents of layer {src}, which has none")
                mx.share(self.mixers[src])

    config_from_dict = staticmethod(MugivikConfig.from_dict)

    def tensor_shapes(self, rank: int = 16) -> dict:
        """Checkpoint names and shapes; rank: of the recurrent layers' decay projections."""
        c = self.config
        C = c.n_embd
        out = {"embed": (c.vocab_size, C), "bigram": (c.buckets + 1, C), "embed.norm": (C,)}
        for i, (mx, ml) in enumerate(zip(self.mixers, self.mlps)):
            sh = mx.shapes(rank) if isinstance(mx, GatedLinearAttention) else mx.shapes()
            out[f"l{i}.norm1"] = (C,)
            out.update({f"l{i}.mix.{k}": s for k, s in sh.items()})
            if ml is not None:
                out[f"l{i}.norm2"] = (C,)
                out.update({f"l{i}.mlp.{k}": s for k, s in ml.shapes().items()})
        out["final.norm"] = (C,)
        return out

    @classmethod
    def from_tensors(cls, config: MugivikConfig, tensors: dict, dtype=torch.bfloat16, device="cuda") -> "Mugivik":
        """The model with the tensors of a checkpoint (names as in tensor_shapes)."""
        if dtype not in (torch.bfloat16, torch.float32):
            raise TypeError(f"Mugivik computes in bfloat16 or float32, not {dtype}")
        m = cls(config)
        m.dtype, m.device = dtype, torch.device(device)
        src = TensorReader(tensors)
        take, group = src.take, src.group

        def vec(name):
            return take(name, (config.n_embd,)).to(device=m.device, dtype=dtype).contiguous()

        C = config.n_embd
        m.Cp = lane_pad(C, dtype)
        # one copy of the table for the lookup and the tied head
        m.embed = m.head = PackedLinear([take("embed", (config.vocab_size, C))], dtype, m.device)
        m.bigram = take("bigram", (config.buckets + 1, C)).to(device=m.device, dtype=dtype).contiguous()
        m.embed_norm, m.final_norm = vec("embed.norm"), vec("final.norm")
        m.norm1, m.norm2 = [], []
        for i, (mx, ml) in enumerate(zip(m.mixers, m.mlps)):
            m.norm1.append(vec(f"l{i}.norm1"))
            mx.load(group(f"l{i}.mix."), dtype, m.device)
            m.norm2.append(None if ml is None else vec(f"l{i}.norm2"))
            if ml is not None:
                ml.load(group(f"l{i}.mlp."), dtype, m.device)
        src.done()
        return m

    @classmethod
    def random(cls, config: MugivikConfig, dtype=torch.bfloat16, device="cuda", seed: int = 1234, rank: int = 16) -> "Mugivik":
        """Random weights of the configuration's shapes (benchmarks, tests)."""
        dev = torch.device(device)
        g = torch.Generator(device=dev).manual_seed(seed)
        t = {}
        for name, shape in cls(config).tensor_shapes(rank).items():
            r = torch.randn(shape, generator=g, device=dev)
            if len(shape) == 1:
                base = 1.0 if name.endswith((".mix.norm", ".dkv.norm")) else 2.0 if name.endswith(".b") else 0.0
                t[name] = base + 0.1 * r
            else:
                t[name] = (r * shape[1] ** -0.5).to(dtype)
        return cls.from_tensors(config, t, dtype, device)

    def new_work(self, M: int, head_rows: int = 0) -> _Work:
        w = _Work(self, M)
        if head_rows:  # before a capture: nothing is allocated by the step itself
            w.head_rows(head_rows, self.Cp, self.dtype)
            for mx in self.mixers:
                mx.reserve(w, M)
        return w

    # ------------------------------------------------------------------ forward over packed rows
    def _embed(self, rows: Rows, w: _Work, state: SequenceState, st) -> None:
        c = self.config
        _hip.call("llj_bigram_embed", rows.tok.data_ptr(), self.embed.w.data_ptr(), self.embed.Kp, self.bigram.data_ptr(),
                  c.n_embd, c.buckets, c.mul_prev, c.mul_cur, self.embed_norm.data_ptr(), c.eps, _hip.ptr(rows.row_seq),
                  _hip.ptr(rows.row0), rows.slot.data_ptr(), state.prev.data_ptr(), rows.pos.data_ptr(), w.x.data_ptr(),
                  self.Cp, None if w.xb is w.x else w.xb.data_ptr(), self.Cp, rows.M, c.n_embd, _dt(self.dtype), st)

    def run(self, rows: Rows, w: _Work, state: SequenceState, logits: torch.Tensor, pick: Optional[torch.Tensor], st,
            taps: Optional[list] = None) -> None:
        """One forward call: logits[i] of row pick[i] (pick None: of every row). `taps`, a list, receives a
        copy of the residual after every layer.

        A sublayer leaves its output in w.t with its norm pending; the next product over the residual
        closes it, in its own launch for one row (PackedLinear.apply_post) or in one before it."""
        M, C, eps = rows.M, self.config.n_embd, self.config.eps
        self._embed(rows, w, state, st)
        x, pending = w.x, None

        def close():
            nonlocal pending
            xb = None if w.xb is w.x else w.xb.data_ptr()
            _hip.call("llj_post_norm", w.t.data_ptr(), self.Cp, pending.data_ptr(), eps, x.data_ptr(), self.Cp, xb, self.Cp,
                      None, None, M, C, _dt(self.dtype), st)
            pending = None

        def product(lin, out, relu2=False):
            nonlocal x, pending
            if pending is not None and lin.takes_post(M, C) and taps is None:
                other = w.x2 if x is w.x else w.x
                lin.apply_post(w.t, pending, eps, x, other, out, st, relu2)
                x, pending = other, None
                return
            if pending is not None:
                close()
            lin.apply(w.xb, M, out, st, relu2)

        for i, (mx, ml) in enumerate(zip(self.mixers, self.mlps)):
            y = w.y[mx.out_width()]
            product(mx.inp, w.proj)
            mx.mix(i, rows, w, state, y, st)
            mx.out.apply(y, M, w.t, st)
            pending = self.norm1[i]
            if ml is not None:
                product(ml.up, w.h, relu2=True)
                ml.down.apply(w.h, M, w.t, st)
                pending = self.norm2[i]
            if taps is not None:
                norm = pending
                close()
                taps.append(w.x[:, :C].clone())
                if i == self.config.n_layer - 1:  # closed already: nothing is left for the head to add
                    w.t.zero_()
                    pending = norm
        n = M if pick is None else pick.numel()
        if n:
            hb, rows_idx = w.head_rows(n, self.Cp, self.dtype), w.all_rows if pick is None else pick
            _hip.call("llj_post_norm", w.t.data_ptr(), self.Cp, pending.data_ptr(), eps, x.data_ptr(), self.Cp, hb.data_ptr(),
                      self.Cp, self.final_norm.data_ptr(), rows_idx.data_ptr(), n, C, _dt(self.dtype), st)
            self.embed.apply(hb, n, logits, st)
        if not rows.decode:
            for i, mx in enumerate(self.mixers):
                if isinstance(mx, LatentAttention):
                    mx.commit(i, rows, w, state, st)
            _hip.call("llj_prev_commit", rows.tok.data_ptr(), rows.row0.data_ptr(), rows.slot.data_ptr(),
                      state.prev.data_ptr(), rows.B, st)
