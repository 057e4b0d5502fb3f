"""Layer mechanisms shared by hybrid models: packed Linear groups, gated linear attention, latent attention,
grouped-query attention, and the squared-relu and clamped gated feed-forwards. Each mixer reads one activation row per token and leaves its gated
output for its output projection; sizes and constants are parameters, the compute is the library's.

Activation type: bfloat16 or float32; the residual, norms, gates of the recurrence, recurrent state and
attention scores are fp32 in both (the kernels' business).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch

from . import _hip
from .state import ALL_POSITIONS
from .utils import find_multiple

GEMM_MIN_ROWS = 64  # bf16: from this many rows on the tiled prefill GEMM, below it slices of STREAM_ROWS
STREAM_ROWS = 16
GLA_CHUNK_RANK = 240  # largest decay rank the chunked recurrence stages
GLA_CHUNK_MIN = 16  # prompts with a sequence longer than this take the chunked recurrence
ATTEND_WGS = 128  # latent decode attention: workgroups the visible keys of a batch are split for (one row: twice)
STREAMS_COLUMNS = 16384  # widest product that also updates the residual streams (7B gated unit, 26112: 61 us against 46 + 4.5)
GQA_WGS = 512  # grouped-query decode attention: workgroups the keys of a batch are split for
GQA_RANGE = 128  # its shortest key range
GQA_LONG = 1024  # prompts with a sequence this long take 128 queries per workgroup where that leaves at least
GQA_WIDE_WGS = 256  # this many workgroups
PART_ALIGN = 8  # output columns of the parts of a packed group start at multiples of this


def _dt(dtype) -> int:
    return 0 if dtype == torch.bfloat16 else 1


def lane_pad(n: int, dtype) -> int:
    """Width of an activation row / a weight's K in memory: the tiled bf16 kernels read 128-deep chunks."""
    return find_multiple(n, 128 if dtype == torch.bfloat16 else 8)


class PackedLinear:
    """Linear layers over the same input as one weight: rows of `parts` stacked (each part's first row
    at a multiple of PART_ALIGN), zero rows and columns up to the kernels' tiles. `offset[i]` is part i's
    first output column. `biases`: one per part (None: none). `unit` = (limit, alpha): two parts of equal size, gate
    and up, interleaved row by row, and the output is their clamped gated unit -- one column per pair, the
    first lane_pad(part rows) columns."""

    def __init__(self, parts: list, dtype, device, biases: Optional[list] = None, unit: Optional[tuple] = None):
        if unit is not None:
            biases = biases or [None, None]
            n, pad = parts[0].shape[0], lane_pad(parts[0].shape[0], dtype)
            if len(parts) != 2 or parts[1].shape != parts[0].shape:
                raise ValueError("a gated unit takes two parts of one shape")
            both = torch.zeros(pad, 2, parts[0].shape[1], dtype=parts[0].dtype, device=parts[0].device)
            bb = torch.zeros(pad, 2, dtype=torch.float32)
            for j, (p, b) in enumerate(zip(parts, biases)):
                both[:n, j] = p
                if b is not None:
                    bb[:n, j] = b.float().cpu()
            parts, biases = [both.view(2 * pad, -1)], [bb.view(-1)]
        self.unit = unit
        self.K = parts[0].shape[1]
        self.Kp = lane_pad(self.K, dtype)
        self.offset, n = [], 0
        for p in parts:
            if p.dim() != 2 or p.shape[1] != self.K:
                raise ValueError(f"packed Linear parts must share their input width, got {[tuple(q.shape) for q in parts]}")
            self.offset.append(n)
            n = find_multiple(n + p.shape[0], PART_ALIGN)
        self.N = self.offset[-1] + parts[-1].shape[0]
        self.Np = lane_pad(self.N, dtype)
        self.dtype = dtype
        self.w = torch.zeros(self.Np, self.Kp, dtype=dtype, device=device)
        for o, p in zip(self.offset, parts):
            self.w[o:o + p.shape[0], :self.K] = p.to(device=device, dtype=dtype)
        self.bias = None
        if biases is not None and any(b is not None for b in biases):
            v = torch.zeros(self.Np, dtype=torch.float32)
            for o, p, b in zip(self.offset, parts, biases):
                if b is not None:
                    v[o:o + p.shape[0]] = b.float().cpu()
            self.bias = v.to(device)
        self.out_columns = self.Np // 2 if unit is not None else self.Np

    def nbytes(self) -> int:
        return self.w.numel() * self.w.element_size()

    def apply(self, a: torch.Tensor, M: int, out: torch.Tensor, st, relu2: bool = False) -> None:
        """out[m, :out_columns] = a[m] . W^T + bias for M rows (padding columns come out zero), through the gated unit,
        or (layers without a bias) max(., 0)^2."""
        if a.shape[1] < self.Kp or out.shape[1] < self.out_columns or a.shape[0] < M or out.shape[0] < M:
            raise ValueError(f"Linear ({self.Np}, {self.Kp}) on a {tuple(a.shape)} into {tuple(out.shape)}, {M} rows")
        limit, alpha = self.unit or (0.0, 0.0)
        act, bias = (2 if self.unit else int(relu2)), _hip.ptr(self.bias)
        if self.dtype == torch.float32:
            y = torch.empty(M, self.Np, dtype=torch.float32, device=out.device) if self.unit else out
            _hip.call("llj_g_linear", 1, a.data_ptr(), a.stride(0), M, self.Kp, self.w.data_ptr(), None, None, 16, self.Kp,
                      self.Np, y.data_ptr(), y.stride(0), None, 0, 1, st)
            if self.unit:
                _hip.call("llj_g_bias_act", 2, y.data_ptr(), y.stride(0), bias, out.data_ptr(), out.stride(0), M, self.Np,
                          limit, alpha, 1, st)
            elif self.bias is not None:
                _hip.call("llj_g_bias_act", 0, y.data_ptr(), y.stride(0), bias, None, 0, M, self.Np, 0.0, 0.0, 1, st)
            if relu2:
                _hip.call("llj_g_relu2", out.data_ptr(), M * out.stride(0), 1, st)
        elif M < GEMM_MIN_ROWS:  # weight-streaming rows
            for r in range(0, M, STREAM_ROWS):
                _hip.call("llj_rows_linear", act, a[r].data_ptr(), a.stride(0), self.w.data_ptr(), bias, out[r].data_ptr(),
                          out.stride(0), min(STREAM_ROWS, M - r), self.Np, self.Kp, limit, alpha, st)
        else:
            nb = 0 if act else _hip.lib().llj_gemm_bf16_ws_bytes(M, self.Np, self.Kp)
            ws = torch.empty(nb // 4, dtype=torch.float32, device=out.device) if nb else None
            _hip.call("llj_gemm_bf16", act, a.data_ptr(), a.stride(0), self.w.data_ptr(), bias, out.data_ptr(),
                      out.stride(0), M, self.Np, self.Kp, limit, alpha, _hip.ptr(ws), nb, st)

    def takes_post(self, M: int, width: int) -> bool:
        """Whether apply_post serves these rows."""
        return self.dtype == torch.bfloat16 and M == 1 and width == self.K and width % 8 == 0 and width <= 8192

    def apply_post(self, t: torch.Tensor, norm: torch.Tensor, eps: float, x: torch.Tensor, x_out: torch.Tensor,
                   out: torch.Tensor, st, relu2: bool = False) -> None:
        """One row: x_out = x + norm(t) and out = x_out . W^T in one launch."""
        _hip.call("llj_post_linear", int(relu2), t.data_ptr(), norm.data_ptr(), eps, x.data_ptr(), x_out.data_ptr(), self.K,
                  self.w.data_ptr(), out.data_ptr(), self.Np, self.Kp, st)


    def takes_streams(self, M: int, width: int, streams: int) -> bool:
        """Whether apply_streams serves these rows (every workgroup of the product reads all streams: with many
        columns a launch of their own is faster)."""
        return (self.dtype == torch.bfloat16 and M == 1 and width == self.K and self.Np <= STREAMS_COLUMNS and
                bool(_hip.lib().llj_streams_linear_ok(streams, width)))

    def apply_streams(self, y: torch.Tensor, done, x: torch.Tensor, x_out: torch.Tensor, sub, eps: float, out: torch.Tensor,
                      st) -> None:
        """One row: the streams after sublayer `done` with its output y (x to x_out), read through sublayer `sub`'s
        weights and norm, then this product, in one launch."""
        limit, alpha = self.unit or (0.0, 0.0)
        _hip.call("llj_streams_linear", 2 if self.unit else 0, y.data_ptr(), done.out.data_ptr(), done.mix.data_ptr(),
                  x.data_ptr(), x_out.data_ptr(), x.shape[-1], x.shape[-2], sub.inp.data_ptr(), sub.norm.data_ptr(), eps,
                  self.K, self.w.data_ptr(), _hip.ptr(self.bias), out.data_ptr(), self.Np, self.Kp, limit, alpha, st)


def rotation_turns(dims: int, base: float, device, factor: float = 1.0) -> torch.Tensor:
    """Frequencies base^(-2i / dims) / factor of a rotation's pairs in turns per position, double precision."""
    i = torch.arange(0, dims, 2, dtype=torch.float64)
    f = torch.pow(torch.tensor(float(base), dtype=torch.float64), -i / dims) / factor
    return (f / (2.0 * torch.pi)).to(device)


# ------------------------------------------------------------------------------------ gated linear attention
@dataclass(frozen=True)
class GLASpec:
    heads: int
    dim: int
    vdim: int
    tau: float


class GatedLinearAttention:
    """S_t = diag(alpha_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t per head, alpha = sigmoid(z)^(1 / tau) per key
    channel with z from a low-rank projection; o RMS-normed per head, gated by silu (csrc/gla.hip)."""

    NAMES = ("q", "k", "v", "g", "o", "norm", "a1", "a2", "a2.b")

    def __init__(self, spec: GLASpec, width: int, eps: float):
        self.spec, self.width, self.eps = spec, width, eps

    def shapes(self, rank: int) -> dict:
        s, C = self.spec, self.width
        HD, HV = s.heads * s.dim, s.heads * s.vdim
        return {"q": (HD, C), "k": (HD, C), "v": (HV, C), "g": (HV, C), "o": (C, HV), "norm": (s.vdim,), "a1": (rank, C),
                "a2": (HD, rank), "a2.b": (HD,)}

    def load(self, t: dict, dtype, device) -> None:
        """t: this mixer's tensors by their names."""
        self.rank = t["a1"].shape[0]
        _check_shapes(t, self.shapes(self.rank))
        self.inp = PackedLinear([t["q"], t["k"], t["v"], t["g"], t["a1"]], dtype, device)
        self.out = PackedLinear([t["o"]], dtype, device)
        self.norm = t["norm"].to(device=device, dtype=dtype).contiguous()
        self.a2 = t["a2"].to(device=device, dtype=dtype).contiguous()
        self.a2b = t["a2.b"].to(device=device, dtype=dtype).contiguous()
        self.dtype = dtype

    def linears(self) -> list:
        return [self.inp, self.out]

    def state_shape(self):
        return self.spec.heads, self.spec.dim, self.spec.vdim

    def ring_window(self):
        return None

    def out_width(self) -> int:
        return self.spec.heads * self.spec.vdim

    def reserve(self, w, M: int) -> None:
        """Scratch of decode steps over M rows (allocated before a step is captured)."""

    def mix(self, i: int, rows, w, state, y: torch.Tensor, st) -> None:
        """y = gated output of layer i from the packed projections w.proj; advances the state."""
        s, p, o = self.spec, w.proj, self.inp.offset
        C = 0
        if not rows.decode and max(rows.lengths) > GLA_CHUNK_MIN and self.rank <= GLA_CHUNK_RANK:
            C = _hip.lib().llj_gla_chunk_rows(s.dim, s.vdim)
        if C:
            n, chunks, first = rows.chunks(C)
            A = torch.empty(rows.M, s.heads * s.dim, dtype=torch.float32, device=p.device)
            U = torch.empty(n, s.heads, s.dim, s.vdim, dtype=torch.float32, device=p.device)
            _hip.call("llj_gla_chunks", p.data_ptr(), p.stride(0), o[0], o[1], o[2], o[3], o[4], self.a2.data_ptr(),
                      self.rank, self.a2b.data_ptr(), self.rank, self.norm.data_ptr(), y.data_ptr(), y.stride(0),
                      state.recurrent[i].data_ptr(), rows.slot.data_ptr(), chunks.data_ptr(), n, first.data_ptr(), rows.B,
                      A.data_ptr(), U.data_ptr(), s.heads, s.dim, s.vdim, s.dim ** -0.5, 1.0 / s.tau, self.eps,
                      _dt(self.dtype), st)
            return
        _hip.call("llj_gla_scan", p.data_ptr(), p.stride(0), o[0], o[1], o[2], o[3], o[4], self.a2.data_ptr(), self.rank,
                  self.a2b.data_ptr(), self.rank, self.norm.data_ptr(), y.data_ptr(), y.stride(0),
                  state.recurrent[i].data_ptr(), _hip.ptr(rows.row0), rows.slot.data_ptr(), rows.B, s.heads, s.dim, s.vdim,
                  s.dim ** -0.5, 1.0 / s.tau, self.eps, _dt(self.dtype), st)


# ------------------------------------------------------------------------------------ latent attention
@dataclass(frozen=True)
class LatentSpec:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    window: int  # a query sees its own and the window - 1 keys before
    scale: float
    rot_base: float
    kv_from: Optional[int] = None  # the layer whose latents this one reads (None: its own)


class LatentAttention:
    """Attention over one RMS-normed latent and one rotated key part per token, sliding window, sigmoid
    output gate (csrc/latent.hip). `kv_from`: reads another layer's latents and has no projection for them."""

    def __init__(self, spec: LatentSpec, width: int, eps: float):
        self.spec, self.width, self.eps = spec, width, eps
        self.owner: Optional[LatentAttention] = None  # whose latents this layer reads (itself by default)
        self.window = spec.window  # the widest window among the layers that read this one's latents

    def share(self, owner: "LatentAttention") -> None:
        a, b = self.spec, owner.spec
        if owner.spec.kv_from is not None:
            raise ValueError("kv_from must name a layer with latents of its own")
        if (a.kv_rank, a.rot_dim, a.rot_base) != (b.kv_rank, b.rot_dim, b.rot_base):
            raise ValueError("layers that share latents must agree in kv_rank, rot_dim and rotation")
        self.owner = owner
        owner.window = max(owner.window, a.window)

    def shapes(self) -> dict:
        s, C = self.spec, self.width
        out = {"q": (s.heads * (s.dim + s.rot_dim), C), "uk": (s.heads * s.dim, s.kv_rank),
               "uv": (s.heads * s.vdim, s.kv_rank), "g": (s.heads * s.vdim, C), "o": (C, s.heads * s.vdim)}
        if s.kv_from is None:
            out.update({"dkv": (s.kv_rank + s.rot_dim, C), "dkv.norm": (s.kv_rank,)})
        return out

    def load(self, t: dict, dtype, device) -> None:
        _check_shapes(t, self.shapes())
        s = self.spec
        own = s.kv_from is None
        self.inp = PackedLinear([t["q"], t["g"]] + ([t["dkv"]] if own else []), dtype, device)
        self.out = PackedLinear([t["o"]], dtype, device)
        self.up = PackedLinear([t["uk"], t["uv"]], dtype, device)
        self.kv_norm = t["dkv.norm"].to(device=device, dtype=dtype).contiguous() if own else None
        self.turns = rotation_turns(s.rot_dim, s.rot_base, device)
        self.dtype = dtype
        if dtype == torch.bfloat16:  # decode rows absorb W_uk into the query: per head [latent column][dim], padded
            self.ukt = torch.zeros(s.heads, self.latent_pad(dtype), find_multiple(s.dim, 32), dtype=dtype, device=device)
            uk = t["uk"].to(device=device, dtype=dtype).view(s.heads, s.dim, s.kv_rank)
            self.ukt[:, :s.kv_rank, :s.dim] = uk.transpose(1, 2)

    def linears(self) -> list:
        return [self.inp, self.up, self.out]

    def state_shape(self):
        return None

    def ring_window(self):
        return self.window if self.spec.kv_from is None else None

    def latent_pad(self, dtype) -> int:
        return lane_pad(self.spec.kv_rank, dtype)

    def cache_width(self, dtype) -> int:
        """Elements of a cached token: the latent up to the tiled K, then the rotated key part."""
        return self.latent_pad(dtype) + find_multiple(self.spec.rot_dim, 8)

    def out_width(self) -> int:
        return self.spec.heads * self.spec.vdim

    def _splits(self, M: int, W: int) -> int:
        s = self.spec
        tiles = (min(s.window, W) + 63) // 64
        wgs = ATTEND_WGS if M > 1 else 2 * ATTEND_WGS
        return max(1, min(tiles, 64, wgs // (M * ((s.heads + 15) // 16))))

    def _decode_ok(self) -> bool:
        s = self.spec
        return (self.dtype == torch.bfloat16 and s.scale > 0 and
                bool(_hip.lib().llj_latent_decode_ok(s.dim, s.rot_dim, self.latent_pad(self.dtype), self.cache_width(self.dtype))))

    def reserve(self, w, M: int) -> None:
        if self._decode_ok():
            s = self.spec
            w.buffer("qc", M * s.heads * self.cache_width(self.dtype), torch.bfloat16)
            w.buffer("part", M * s.heads * self._splits(M, s.window) * (self.latent_pad(self.dtype) + 4), torch.float32)

    def mix(self, i: int, rows, w, state, y: torch.Tensor, st) -> None:
        s, p = self.spec, w.proj
        own = s.kv_from is None
        src = i if own else s.kv_from
        ring, W = state.ring[src], state.ring_rows[src]
        o, M = self.inp.offset, rows.M
        okv = o[2] if own else -1
        krp, ldc = self.latent_pad(self.dtype), self.cache_width(self.dtype)
        up = self.up
        if rows.decode and self._decode_ok():
            n = self._splits(M, W)
            qc = w.buffer("qc", M * s.heads * ldc, torch.bfloat16)
            part = w.buffer("part", M * s.heads * n * (krp + 4), torch.float32)
            _hip.call("llj_latent_decode", p.data_ptr(), p.stride(0), o[0], o[1], okv, self.ukt.data_ptr(),
                      up.w[up.offset[1]:].data_ptr(), _hip.ptr(self.kv_norm), self.turns.data_ptr(), rows.pos.data_ptr(), rows.slot.data_ptr(),
                      ring.data_ptr(), W, s.window, qc.data_ptr(), part.data_ptr(), n, y.data_ptr(), y.stride(0), M, s.heads,
                      s.dim, s.rot_dim, s.vdim, s.kv_rank, krp, ldc, self.eps, s.scale, st)
            return
        if own and not rows.decode:
            w.cur[i] = torch.empty(M, ldc, dtype=self.dtype, device=p.device)
        cur = None if rows.decode else w.cur[src]
        _hip.call("llj_latent_prep", p.data_ptr(), p.stride(0), o[0], okv, _hip.ptr(self.kv_norm), self.turns.data_ptr(),
                  rows.pos.data_ptr(), rows.slot.data_ptr(), _hip.ptr(cur), ring.data_ptr(), W, M, s.heads, s.dim, s.rot_dim,
                  s.kv_rank, krp, ldc, self.eps, _dt(self.dtype), st)
        if (not rows.decode and self.dtype == torch.bfloat16 and s.scale > 0 and
                _hip.lib().llj_latent_flash_ok(s.dim, s.rot_dim, s.vdim)):
            nk, gather, key0, kpos0, nkey = rows.keys(s.window)
            lat = cur
            if gather is not None:
                lat = torch.empty(nk, ldc, dtype=self.dtype, device=p.device)
                _hip.call("llj_latent_gather", cur.data_ptr(), ring.data_ptr(), W, ldc, gather[0].data_ptr(),
                          gather[1].data_ptr(), gather[2].data_ptr(), lat.data_ptr(), nk, st)
            kv = torch.empty(nk, up.Np, dtype=self.dtype, device=p.device)
            up.apply(lat, nk, kv, st)
            n, chunks, _ = rows.chunks(64)
            _hip.call("llj_latent_flash", p.data_ptr(), p.stride(0), o[0], o[1], kv.data_ptr(), kv.stride(0), up.offset[1],
                      lat.data_ptr(), ldc, krp, chunks.data_ptr(), n, rows.pos.data_ptr(), key0.data_ptr(),
                      kpos0.data_ptr(), nkey.data_ptr(), y.data_ptr(), y.stride(0), s.window, s.heads, s.dim, s.rot_dim,
                      s.vdim, s.scale, st)
            return
        uv = up.w[up.offset[1]:]
        _hip.call("llj_latent_rows", p.data_ptr(), p.stride(0), o[0], o[1], up.w.data_ptr(), up.Kp, uv.data_ptr(), up.Kp,
                  _hip.ptr(cur), ring.data_ptr(), W, s.window, _hip.ptr(rows.row_seq), _hip.ptr(rows.row0),
                  rows.pos.data_ptr(), rows.slot.data_ptr(), y.data_ptr(), y.stride(0), M, s.heads, s.dim, s.rot_dim, s.vdim,
                  s.kv_rank, krp, ldc, s.scale, _dt(self.dtype), st)

    def commit(self, i: int, rows, w, state, st) -> None:
        """After the last layer of a prompt call: the new tokens' latents into the ring."""
        if self.spec.kv_from is None:
            _hip.call("llj_latent_commit", w.cur[i].data_ptr(), state.ring[i].data_ptr(), state.ring_rows[i],
                      self.cache_width(self.dtype), rows.row_seq.data_ptr(), rows.row0.data_ptr(), rows.pos.data_ptr(),
                      rows.slot.data_ptr(), rows.M, _dt(self.dtype), st)


# ------------------------------------------------------------------------------------ grouped-query attention
@dataclass(frozen=True)
class GroupedSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int
    rot_base: float
    rot_factor: float = 1.0  # divides the rotation's frequencies
    v_mix: bool = False  # values mixed with those of the first such layer
    qk_norm: bool = True  # rotated queries and keys divided by their root mean square
    sink: bool = True  # a key of score 0 without a value


class GroupedAttention:
    """Causal grouped-query attention with biased projections, rotate-half positions and one sigmoid gate per
    head (csrc/gqa.hip). Keeps a K / V row of every token (state.ALL_POSITIONS)."""

    def __init__(self, spec: GroupedSpec, width: int, eps: float):
        self.spec, self.width, self.eps = spec, width, eps
        self.first: Optional[GroupedAttention] = None  # v_mix: the layer whose values are mixed in (itself: it leaves them)

    def shapes(self) -> dict:
        s, C = self.spec, self.width
        out = {"q": (s.heads * s.dim, C), "k": (s.kv_heads * s.dim, C), "v": (s.kv_heads * s.vdim, C), "g": (s.heads, C),
               "o": (C, s.heads * s.vdim)}
        out.update({n + ".b": (out[n][0],) for n in "qkvo"})
        if s.v_mix:
            out["vmix"] = ()
        return out

    def load(self, t: dict, dtype, device) -> None:
        s = self.spec
        if not s.v_mix:
            t.pop("vmix", None)
        _check_shapes(t, self.shapes())
        self.inp = PackedLinear([t["q"], t["k"], t["v"], t["g"]], dtype, device, [t["q.b"], t["k.b"], t["v.b"], None])
        self.out = PackedLinear([t["o"]], dtype, device, [t["o.b"]])
        self.lam = t["vmix"].to(device=device, dtype=torch.float32).reshape(1) if s.v_mix and self.first is not self else None
        self.turns = rotation_turns(s.rot_dims, s.rot_base, device, s.rot_factor)
        self.dtype = dtype

    def linears(self) -> list:
        return [self.inp, self.out]

    def state_shape(self):
        return None

    def ring_window(self):
        return ALL_POSITIONS

    def cache_width(self, dtype) -> int:
        return find_multiple(self.spec.kv_heads * (self.spec.dim + self.spec.vdim), 8)

    def out_width(self) -> int:
        return self.spec.heads * self.spec.vdim

    def first_width(self) -> int:
        """Columns of the values the first mixing layer leaves for the others."""
        return self.spec.kv_heads * self.spec.vdim if self.spec.v_mix else 0

    def _decode_ok(self) -> bool:
        s = self.spec
        return self.dtype == torch.bfloat16 and bool(_hip.lib().llj_gqa_decode_ok(s.dim, s.vdim))

    def _splits(self, M: int, W: int) -> int:
        """Key ranges of a decode step over a cache of W rows (None: the most there can be)."""
        s = self.spec
        most = max(1, min(64, GQA_WGS // (M * s.kv_heads * ((s.heads // s.kv_heads + 15) // 16))))
        if W is None:
            return most
        n = -(-W // GQA_RANGE)
        return min(most, n if n <= 8 else max(8, -(-W // (2 * GQA_RANGE))))

    def _part(self, w, M: int, n: int):
        """Partials and counters of a decode step's key ranges (the counters start at zero, and every step leaves them so)."""
        s = self.spec
        return (w.buffer("part", M * s.heads * n * _hip.lib().llj_gqa_part_width(s.vdim), torch.float32),
                w.buffer("count", M * s.heads, torch.int32, zero=True))

    def reserve(self, w, M: int) -> None:
        if self._decode_ok():
            self._part(w, M, self._splits(M, None))

    def mix(self, i: int, rows, w, state, y: torch.Tensor, st) -> None:
        """y = gated output of layer i from the packed projections w.proj; the rows' keys and values into the state."""
        s, p, o, M = self.spec, w.proj, self.inp.offset, rows.M
        cache, W, ldc = state.ring[i], state.ring_rows[i], self.cache_width(self.dtype)
        first = w.first if s.v_mix else None
        new = (self.turns.data_ptr(), s.rot_dims, int(s.qk_norm), self.eps)
        mixed = (_hip.ptr(first), _hip.ptr(self.lam), 0 if first is None else first.stride(0))
        sizes = (M, s.heads, s.kv_heads, s.dim, s.vdim)
        if rows.decode and self._decode_ok():
            n = self._splits(M, W)
            _hip.call("llj_gqa_decode", p.data_ptr(), p.stride(0), o[0], o[1], o[2], o[3], *new, rows.pos.data_ptr(),
                      rows.slot.data_ptr(), cache.data_ptr(), W, ldc, *mixed, *(t.data_ptr() for t in self._part(w, M, n)), n,
                      y.data_ptr(), y.stride(0), *sizes, s.scale, int(s.sink), st)
            return
        _hip.call("llj_gqa_prep", p.data_ptr(), p.stride(0), o[0], o[1], o[2], *new, rows.pos.data_ptr(),
                  _hip.ptr(rows.row_seq), rows.slot.data_ptr(), cache.data_ptr(), W, ldc, *mixed, *sizes, _dt(self.dtype), st)
        C = 0
        if not rows.decode and self.dtype == torch.bfloat16:
            wide = s.heads * sum(-(-n // 256) for n in rows.lengths)  # workgroups of two 128-query blocks
            C = _hip.lib().llj_gqa_flash_rows(s.dim, s.vdim, int(max(rows.lengths) >= GQA_LONG and wide >= GQA_WIDE_WGS))
        if C:
            n, work = rows.pairs(C)
            _hip.call("llj_gqa_flash", p.data_ptr(), p.stride(0), o[0], o[3], work.data_ptr(), n, C, rows.pos.data_ptr(),
                      rows.slot.data_ptr(), cache.data_ptr(), W, ldc, y.data_ptr(), y.stride(0), *sizes, s.scale,
                      int(s.sink), st)
            return
        _hip.call("llj_gqa_rows", p.data_ptr(), p.stride(0), o[0], o[3], rows.pos.data_ptr(), _hip.ptr(rows.row_seq),
                  rows.slot.data_ptr(), cache.data_ptr(), W, ldc, y.data_ptr(), y.stride(0), *sizes, s.scale, int(s.sink),
                  _dt(self.dtype), st)


# ------------------------------------------------------------------------------------ feed-forward
class ReluSquaredMLP:
    """W_down max(W_up h, 0)^2"""

    def __init__(self, ff: int, width: int):
        self.ff, self.width = ff, width

    def shapes(self) -> dict:
        return {"up": (self.ff, self.width), "down": (self.width, self.ff)}

    def load(self, t: dict, dtype, device) -> None:
        _check_shapes(t, self.shapes())
        self.up = PackedLinear([t["up"]], dtype, device)
        self.down = PackedLinear([t["down"]], dtype, device)

    def linears(self) -> list:
        return [self.up, self.down]


class ClampedGLU:
    """W_down of the clamped gated unit (PackedLinear's `unit`) of W_gate h and W_up h, all biased."""

    def __init__(self, ff: int, width: int, limit: float, alpha: float):
        self.ff, self.width, self.unit = ff, width, (limit, alpha)

    def shapes(self) -> dict:
        F, C = self.ff, self.width
        return {"gate": (F, C), "gate.b": (F,), "up": (F, C), "up.b": (F,), "down": (C, F), "down.b": (C,)}

    def load(self, t: dict, dtype, device) -> None:
        _check_shapes(t, self.shapes())
        self.up = PackedLinear([t["gate"], t["up"]], dtype, device, [t["gate.b"], t["up.b"]], unit=self.unit)
        self.down = PackedLinear([t["down"]], dtype, device, [t["down.b"]])

    def linears(self) -> list:
        return [self.up, self.down]


# ------------------------------------------------------------------------------------ residual streams
@dataclass
class StreamSublayer:
    """How a sublayer reads and leaves the residual streams (csrc/streams.hip): u = sum_s inp[s] x_s through a layer
    norm with weight `norm`, then x_t = sum_s mix[s, t] x_s + out[t] y."""

    inp: torch.Tensor
    out: torch.Tensor
    mix: torch.Tensor
    norm: torch.Tensor


def _check_shapes(t: dict, want: dict) -> None:
    if set(t) != set(want):
        raise ValueError(f"tensors {sorted(set(want) - set(t))} missing, {sorted(set(t) - set(want))} unexpected")
    for k, s in want.items():
        if tuple(t[k].shape) != tuple(s):
            raise ValueError(f"tensor {k} has shape {tuple(t[k].shape)}, expected {tuple(s)}")
