"""Bobasun: a decoder whose residual is several streams (hyper-connections), with grouped-query attention and clamped
gated feed-forwards, bias-free layer norms on the sublayers' inputs and an untied head.

  x_1 = .. = x_s = embed[token] * scale
  per sublayer: y = sublayer(layer_norm(sum_s in[s] x_s)); x_t = sum_s mix[s, t] x_s + out[t] y
  logits = head . layer_norm(sum_s x_s)

The streams are fp32. A forward call takes packed activation rows (state.Rows) like the other models with
per-sequence state. Everything runs on the library's kernels: packed projections (mixers.PackedLinear),
csrc/gqa.hip and csrc/streams.hip; for one row the streams are updated in the next product's launch.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple

import torch

from . import _hip
from .hybrid import MAX_POSITIONS, HybridModel, Scratch, TensorReader, take_values
from .mixers import ClampedGLU, GroupedAttention, GroupedSpec, PackedLinear, StreamSublayer, _dt, lane_pad
from .registry import register
from .state import Rows, SequenceState
from .utils import find_multiple

GLU_ALPHA = 1.702  # the gated unit's sigmoid slope


@dataclass(frozen=True)
class BobasunLayer:
    mixer: GroupedSpec
    ff: Optional[int]  # None: no feed-forward
    limit: float = 0.0


@dataclass(frozen=True)
class BobasunConfig:
    vocab_size: int
    n_embd: int
    eps: float
    embed_scale: float
    streams: int
    layers: Tuple[BobasunLayer, ...]

    block_size = MAX_POSITIONS

    @property
    def padded_vocab_size(self) -> int:
        return find_multiple(self.vocab_size, 128)

    @property
    def n_layer(self) -> int:
        return len(self.layers)

    @classmethod
    def from_dict(cls, d: dict) -> "BobasunConfig":
        _, emb, layers, norm, streams, vocab, width = take_values(
            d, "config.json", architecture=str, embedding=dict, layers=list, norm=dict, streams=int, vocab=int, width=int)
        (scale,) = take_values(emb, "embedding", scale=float)
        (eps,) = take_values(norm, "norm", eps=float)
        out, mixing = [], None
        for i, layer in enumerate(layers):
            where = f"layers[{i}]"
            mix, mlp, kind = take_values(layer, where, mixer=dict, mlp=(dict, None), type=str)
            if kind != "attention":
                raise ValueError(f"config: {where} has unknown type {kind!r}")
            heads, kv, dim, vdim, att_scale, rot, v_mix = take_values(
                mix, where + ".mixer", heads=int, kv_heads=int, dim=int, vdim=int, scale=float, rot=dict, v_mix=(bool, False))
            base, dims, scaling = take_values(rot, where + ".mixer.rot", base=float, dims=int, scaling=(dict, None))
            (factor,) = (1.0,) if scaling is None else take_values(scaling, where + ".mixer.rot.scaling", factor=float)
            if min(heads, kv, dim, vdim) < 1 or heads % kv:
                raise ValueError(f"config: {where} has {heads} query heads on {kv} key / value heads of {dim} and {vdim}")
            if dims % 2 or not 0 <= dims <= dim:
                raise ValueError(f"config: {where} rotates {dims} of {dim} dimensions")
            if v_mix:
                mixing = mixing or (kv, vdim)
                if mixing != (kv, vdim):
                    raise ValueError(f"config: {where} mixes values of {kv} x {vdim} with {mixing[0]} x {mixing[1]}")
            spec = GroupedSpec(heads, kv, dim, vdim, att_scale, dims, base, factor, bool(v_mix))
            ff, limit = None, 0.0
            if mlp is not None:
                ff, mk, limit = take_values(mlp, where + ".mlp", ff=int, kind=str, limit=float)
                if mk != "dense":
                    raise ValueError(f"config: {where}.mlp has unknown kind {mk!r}")
            out.append(BobasunLayer(spec, ff, limit))
        if not out or min(vocab, width, streams) < 1:
            raise ValueError("config: needs at least one layer, a vocabulary, a width and a stream")
        return cls(vocab, width, eps, scale, streams, tuple(out))


class _Work(Scratch):
    def __init__(self, m: "Bobasun", M: int):
        dev, dt, C = m.device, m.dtype, m.Cp
        super().__init__(M, dev)
        self.x = torch.empty(M, m.config.streams, m.config.n_embd, dtype=torch.float32, device=dev)
        self.x2 = torch.empty_like(self.x) if M == 1 else None  # the streams' other place (fused products)
        self.h = torch.empty(M, C, dtype=dt, device=dev)  # a sublayer's normed input
        self.t = torch.empty(M, C, dtype=dt, device=dev)  # and its output
        self.proj = torch.empty(M, max(mx.inp.Np for mx in m.mixers), dtype=dt, device=dev)
        ff = [f.up.out_columns for f in m.mlps if f is not None]
        self.f = torch.empty(M, max(ff), dtype=dt, device=dev) if ff else None
        # mixer outputs by width: padding columns stay zero
        self.y = {n: torch.zeros(M, lane_pad(n, dt), dtype=dt, device=dev) for n in {mx.out_width() for mx in m.mixers}}
        n = max(mx.first_width() for mx in m.mixers)
        self.first = torch.empty(M, n, dtype=dt, device=dev) if n else None  # the first mixing layer's values


@register("Bobasun")
class Bobasun(HybridModel):
    HIP_SOURCES = ("streams", "post_gemv", "gemm_bf16", "gqa", "generic", "ops", "options")

    def __init__(self, config: BobasunConfig):
        super().__init__()
        self.config = config
        C, eps = config.n_embd, config.eps
        self.mixers = [GroupedAttention(layer.mixer, C, eps) for layer in config.layers]
        self.mlps = [None if layer.ff is None else ClampedGLU(layer.ff, C, layer.limit, GLU_ALPHA) for layer in config.layers]
        mixing = [mx for mx in self.mixers if mx.spec.v_mix]
        for mx in mixing:
            mx.first = mixing[0]

    config_from_dict = staticmethod(BobasunConfig.from_dict)

    def tensor_shapes(self) -> dict:
        """Checkpoint names and shapes."""
        c = self.config
        C, S = c.n_embd, c.streams
        out = {"embed": (c.vocab_size, C)}
        for i, (mx, ml) in enumerate(zip(self.mixers, self.mlps)):
            for q, part, shapes in ((1, "mix", mx.shapes()), (2, "mlp", ml and ml.shapes())):
                if shapes is not None:
                    out[f"l{i}.norm{q}"] = (C,)
                    out.update({f"l{i}.{part}.{k}": s for k, s in shapes.items()})
                    out.update({f"l{i}.hc{q}.in": (S,), f"l{i}.hc{q}.out": (S,), f"l{i}.hc{q}.mix": (S, S)})
        out["final.norm"] = (C,)
        out["head"] = (c.vocab_size, C)
        return out

    @classmethod
    def from_tensors(cls, config: BobasunConfig, tensors: dict, dtype=torch.bfloat16, device="cuda") -> "Bobasun":
        """The model with the tensors of a checkpoint (names as in tensor_shapes)."""
        if dtype not in (torch.bfloat16, torch.float32):
            raise TypeError(f"Bobasun computes in bfloat16 or float32, not {dtype}")
        m = cls(config)
        m.dtype, m.device = dtype, torch.device(device)
        src, C, S = TensorReader(tensors), config.n_embd, config.streams
        m.Cp = lane_pad(C, dtype)

        def put(name, shape, kind=dtype):
            return src.take(name, shape).to(device=m.device, dtype=kind).contiguous()

        def sublayer(i, q):
            inp, out, mix = (put(f"l{i}.hc{q}.{n}", s, torch.float32) for n, s in (("in", (S,)), ("out", (S,)), ("mix", (S, S))))
            return StreamSublayer(inp, out, mix, put(f"l{i}.norm{q}", (C,)))

        m.embed = put("embed", (config.vocab_size, C))
        m.subs = []  # per layer: the mixer's place in the streams, the feed-forward's
        for i, (mx, ml) in enumerate(zip(m.mixers, m.mlps)):
            mx.load(src.group(f"l{i}.mix."), dtype, m.device)
            if ml is not None:
                ml.load(src.group(f"l{i}.mlp."), dtype, m.device)
            m.subs.append((sublayer(i, 1), None if ml is None else sublayer(i, 2)))
        m.final_norm = put("final.norm", (C,))
        m.head = PackedLinear([src.take("head", (config.vocab_size, C))], dtype, m.device)
        src.done()
        return m

    @classmethod
    def random(cls, config: BobasunConfig, dtype=torch.bfloat16, device="cuda", seed: int = 1234) -> "Bobasun":
        """Random weights of the configuration's shapes (benchmarks, tests)."""
        dev = torch.device(device)
        g = torch.Generator(device=dev).manual_seed(seed)
        S, t = config.streams, {}
        for name, shape in cls(config).tensor_shapes().items():
            r = torch.randn(shape, generator=g, device=dev)
            if name.endswith(".mix") and ".hc" in name:  # near the identity
                t[name] = torch.eye(S, device=dev) * 0.9 + 0.1 / S + 0.02 * r
            elif ".hc" in name:
                t[name] = (1.0 / S if name.endswith(".in") else 1.0) + 0.1 * r
            elif name.endswith(".vmix"):
                t[name] = 0.4 + 0.1 * r
            elif len(shape) == 1:
                t[name] = (0.0 if name.endswith(".b") else 1.0) + 0.1 * r
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
    def run(self, rows: Rows, w: _Work, state: SequenceState, logits: torch.Tensor, pick: Optional[torch.Tensor], st,
            taps: Optional[list] = None) -> None:
        """One forward call: logits[i] of row pick[i] (pick None: of every row). `taps`, a list, receives the
        sum of the streams after every layer.

        A sublayer leaves its output in w.t with the streams' update pending (`done`); the next sublayer's first
        product closes it, in its own launch for one row (PackedLinear.apply_streams) or in one before it."""
        c, M, C, eps, S, dt = self.config, rows.M, self.config.n_embd, self.config.eps, self.config.streams, _dt(self.dtype)
        x, done = w.x, None
        first = self.subs[0][0]
        _hip.call("llj_streams_embed", rows.tok.data_ptr(), self.embed.data_ptr(), C, c.embed_scale,
                  rows.pos.data_ptr() if rows.decode else None, x.data_ptr(), C, S, first.inp.data_ptr(), first.norm.data_ptr(),
                  eps, w.h.data_ptr(), self.Cp, M, C, dt, st)

        def step(x, inp, norm, h, picked=None, n=M):
            _hip.call("llj_streams_step", w.t.data_ptr(), self.Cp, done.out.data_ptr(), done.mix.data_ptr(), x.data_ptr(), C, S,
                      _hip.ptr(inp), norm.data_ptr(), eps, h.data_ptr(), self.Cp, _hip.ptr(picked), n, C, dt, st)

        def product(lin, sub, out):
            nonlocal x
            if done is not None and lin.takes_streams(M, C, S):
                other = w.x2 if x is w.x else w.x
                lin.apply_streams(w.t, done, x, other, sub, eps, out, st)
                x = other
                return
            if done is not None:
                step(x, sub.inp, sub.norm, w.h)
            lin.apply(w.h, M, out, st)

        for i, (mx, ml, (sub1, sub2)) in enumerate(zip(self.mixers, self.mlps, self.subs)):
            y = w.y[mx.out_width()]
            product(mx.inp, sub1, w.proj)
            mx.mix(i, rows, w, state, y, st)
            mx.out.apply(y, M, w.t, st)
            done = sub1
            if ml is not None:
                product(ml.up, sub2, w.f)
                ml.down.apply(w.f, M, w.t, st)
                done = sub2
            if taps is not None:
                after = x.clone()
                step(after, None, self.final_norm, torch.empty_like(w.h))
                taps.append(after.sum(1))
        n = M if pick is None else pick.numel()
        if n:
            hb = w.head_rows(n, self.Cp, self.dtype)
            step(x, None, self.final_norm, hb, w.all_rows if pick is None else pick, n)
            self.head.apply(hb, n, logits, st)
