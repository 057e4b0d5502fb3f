"""The hybrid models' kernels one by one (csrc/postnorm, post_gemv, gemm_bf16, gla, latent*, streams, gqa) against
the functions of oracle/mugivik_np.py and oracle/bobasun_np.py or plain float64 numpy."""
import numpy as np
import pytest
import torch

from oracle import bobasun_np as B
from oracle import mugivik_np as O

pytestmark = pytest.mark.gpu
DT = {torch.bfloat16: 0, torch.float32: 1}


def dev(a, dtype=torch.float32):
    return torch.as_tensor(np.ascontiguousarray(a)).to(dtype).cuda()


def ints(*a):
    return torch.tensor(a, dtype=torch.int32, device="cuda")


def back(t):
    return t.float().cpu().numpy().astype(np.float64)


def call(name, *args):
    from lit_llama import _hip

    _hip.call(name, *[a.data_ptr() if isinstance(a, torch.Tensor) else a for a in args], _hip.stream())


def close(got, want, rel, what=""):
    s = np.abs(want).max() or 1.0
    e = np.abs(np.asarray(got, np.float64) - want).max() / s
    assert e < rel, f"{what}: {e:.3g} of the largest value, limit {rel}"


@pytest.mark.parametrize("dtype", list(DT))
@pytest.mark.parametrize("C", [8, 72, 75, 2048, 3072, 5120, 8192, 9000])
def test_post_norm(hip, dtype, C):
    g = np.random.default_rng(C)
    M, ld, eps = 5, (C + 7) // 8 * 8 + 8, 1e-5
    t, x = dev(g.standard_normal((M, ld)) * 3, dtype), dev(g.standard_normal((M, ld)))
    w, w2 = dev(0.3 * g.standard_normal(C), dtype), dev(0.3 * g.standard_normal(C), dtype)
    xb = torch.full((M, ld), 7.0, dtype=dtype, device="cuda")
    x0 = x.clone()
    want = back(x0)[:, :C] + O.norm_zero(back(t)[:, :C], back(w), eps)
    rel = 2e-6 if dtype == torch.float32 else 6e-3
    # the last norm of gathered rows leaves x alone
    pick = ints(4, 0, 3)
    hb = torch.empty(3, ld, dtype=dtype, device="cuda")
    call("llj_post_norm", t, ld, w, eps, x, ld, hb, ld, w2, pick, 3, C, DT[dtype])
    assert torch.equal(x, x0)
    close(back(hb)[:, :C], O.norm_zero(want[[4, 0, 3]], back(w2), eps), rel, "gathered")
    call("llj_post_norm", t, ld, w, eps, x, ld, xb, ld, None, None, M, C, DT[dtype])
    close(back(x)[:, :C], want, 2e-6, "residual")
    close(back(xb)[:, :C], want, rel, "copy")
    assert float(xb[:, C:].abs().max()) == 0.0 and torch.equal(x[:, C:], x0[:, C:])


@pytest.mark.parametrize("dtype", list(DT))
def test_bigram_embed(hip, dtype):
    g = np.random.default_rng(0)
    V, C, K, mp, mc, eps = 40, 24, 11, 13, 3, 1e-6
    emb, big, w = dev(g.standard_normal((V, C)), dtype), dev(g.standard_normal((K + 1, C)), dtype), dev(0.2 * g.standard_normal(C), dtype)
    seqs = [[5, 39, 0, 7], [2], [9, 9]]
    cfg = {"embedding": {"bigram": {"buckets": K, "mul_prev": mp, "mul_cur": mc}}, "norm": {"eps": eps}}
    P = {"embed": back(emb), "bigram": back(big), "embed.norm": back(w)}
    want = np.concatenate([O.embedding(s, cfg, P) for s in seqs])
    tok = ints(*[t for s in seqs for t in s])
    slot, prev = ints(2, 0, 3), torch.full((4,), -1, dtype=torch.int32, device="cuda")
    x, xb = torch.zeros(7, 32, device="cuda"), torch.zeros(7, 32, dtype=dtype, device="cuda")
    rel = 2e-6 if dtype == torch.float32 else 6e-3
    call("llj_bigram_embed", tok, emb, C, big, C, K, mp, mc, w, eps, ints(0, 0, 0, 0, 1, 2, 2), ints(0, 4, 5, 7), slot, prev, None,
         x, 32, xb, 32, 7, C, DT[dtype])
    close(back(x)[:, :C], want, 2e-6)
    close(back(xb)[:, :C], want, rel)
    assert prev.tolist() == [-1] * 4
    call("llj_prev_commit", tok, ints(0, 4, 5, 7), slot, prev, 3)
    assert prev.tolist() == [2, -1, 7, 9]
    # decode rows: the state's token is the previous one, and moves on with the position
    pos = ints(3, 0, 1)
    call("llj_bigram_embed", ints(1, 38, 9), emb, C, big, C, K, mp, mc, w, eps, None, None, slot, prev, pos, x, 32, None, 0, 3, C,
         DT[dtype])
    want = np.stack([O.embedding(s + [t], cfg, P)[-1] for s, t in zip(seqs, (1, 38, 9))])
    close(back(x)[:3, :C], want, 2e-6)
    assert prev.tolist() == [38, -1, 1, 9] and pos.tolist() == [4, 1, 2]


@pytest.mark.parametrize("M", [1, 2, 7, 8, 9, 16])
@pytest.mark.parametrize("N,K", [(128, 128), (384, 256), (2048, 2048), (256, 8448), (5632, 1152)])
@pytest.mark.parametrize("act", [0, 1])
def test_rows_linear(hip, M, N, K, act):
    g = torch.Generator(device="cuda").manual_seed(M * N + K)
    A = torch.randn(M, K + 8, generator=g, device="cuda").to(torch.bfloat16)
    W = (torch.randn(N, K, generator=g, device="cuda") * K ** -0.5).to(torch.bfloat16)
    out = torch.full((M, N + 16), 3.0, dtype=torch.bfloat16, device="cuda")
    call("llj_rows_linear", act, A, K + 8, W, None, out, N + 16, M, N, K, 0.0, 0.0)
    want = back(A)[:, :K] @ back(W).T
    want = np.maximum(want, 0) ** 2 if act else want
    close(back(out)[:, :N], want, 5e-3)
    assert float((out[:, N:] - 3.0).abs().max()) == 0.0


@pytest.mark.parametrize("C,K,N", [(72, 128, 256), (2048, 2048, 384), (4096, 4096, 128), (8192, 8192, 4224), (1000, 1024, 8448)])
@pytest.mark.parametrize("act", [0, 1])
def test_post_linear(hip, C, K, N, act):
    g = np.random.default_rng(C + N)
    t, w, x = dev(2 * g.standard_normal(C), torch.bfloat16), dev(0.3 * g.standard_normal(C), torch.bfloat16), dev(g.standard_normal(C))
    W = dev(g.standard_normal((N, K)) * C ** -0.5, torch.bfloat16)
    xo = torch.zeros(C, device="cuda")
    out = torch.empty(N, dtype=torch.bfloat16, device="cuda")
    call("llj_post_linear", act, t, w, 1e-5, x, xo, C, W, out, N, K)
    xn = back(x) + O.norm_zero(back(t), back(w), 1e-5)
    close(back(xo), xn, 2e-6)
    y = xn @ back(W)[:, :C].T
    close(back(out), np.maximum(y, 0) ** 2 if act else y, 1.2e-2)


@pytest.mark.parametrize("M", [64, 100, 256, 300, 1024])
@pytest.mark.parametrize("N,K", [(128, 128), (2048, 1024), (384, 2048)])
@pytest.mark.parametrize("act", [0, 1])
def test_gemm_bf16(hip, M, N, K, act):
    from lit_llama import _hip

    g = torch.Generator(device="cuda").manual_seed(M + N + K)
    A = torch.randn(M, K, generator=g, device="cuda").to(torch.bfloat16)
    W = (torch.randn(N, K, generator=g, device="cuda") * K ** -0.5).to(torch.bfloat16)
    out = torch.empty(M, N, dtype=torch.bfloat16, device="cuda")
    nb = _hip.lib().llj_gemm_bf16_ws_bytes(M, N, K)
    want = back(A) @ back(W).T
    want = np.maximum(want, 0) ** 2 if act else want
    for ws in {None, nb or None}:
        buf = None if ws is None else torch.empty(nb // 4, device="cuda")
        call("llj_gemm_bf16", act, A, K, W, None, out, N, M, N, K, 0.0, 0.0, buf, nb)
        close(back(out), want, 5e-3, ws)


def _gla_case(g, lens, H, D, V, rank, dtype, bias=None):
    M, HD, HV = sum(lens), H * D, H * V
    off = np.cumsum([0, HD, HD, HV, HV])
    ld = int(off[-1]) + rank + 3
    inp = g.standard_normal((M, ld))
    a2, b = g.standard_normal((HD, rank)) * rank ** -0.5, g.uniform(-3, 5, HD) if bias is None else bias
    return [int(o) for o in off], ld, dev(inp, dtype), dev(a2, dtype), dev(b, dtype), dev(1 + 0.2 * g.standard_normal(V), dtype)


def _gla_ref(off, inp, a2, b, nw, lens, H, D, V, tau, eps, S0):
    x, out, S = back(inp), [], S0.copy()
    loga = -np.logaddexp(0.0, -(x[:, off[4]:off[4] + a2.shape[1]] @ back(a2).T + back(b))) / tau
    r = 0
    for s, n in enumerate(lens):
        rows = slice(r, r + n)
        y = np.empty((n, H * V))
        for h in range(H):
            q, k = (x[rows, off[i] + h * D:off[i] + (h + 1) * D] for i in (0, 1))
            v, gt = (x[rows, off[i] + h * V:off[i] + (h + 1) * V] for i in (2, 3))
            o, S[s, h] = O.gla_recurrence(q * D ** -0.5, k, v, loga[rows, h * D:(h + 1) * D], S[s, h])
            y[:, h * V:(h + 1) * V] = O.rms(o, eps) * back(nw) * O.silu(gt)
        out.append(y)
        r += n
    return np.concatenate(out), S


@pytest.mark.parametrize("dtype", list(DT))
@pytest.mark.parametrize("H,D,V,rank", [(2, 64, 128, 16), (3, 12, 20, 5), (1, 1, 1, 1), (2, 48, 96, 8), (1, 256, 64, 24), (2, 33, 510, 16),
                                        (1, 128, 256, 20)])
@pytest.mark.parametrize("form", ["scan", "chunks"])
def test_gla(hip, form, dtype, H, D, V, rank):
    """Token by token and in chunks, from states that are not zero, sequences of unequal lengths and other slots."""
    from lit_llama import _hip
    from lit_llama.state import Rows

    g = np.random.default_rng(D * V)
    lens, slots, tau, eps = [70, 1, 130, 64], [3, 0, 4, 1], 2.0, 1e-5
    off, ld, inp, a2, b, nw = _gla_case(g, lens, H, D, V, rank, dtype)
    S0 = g.standard_normal((4, H, D, V))
    state = torch.full((5, H, D, V), 9.0, device="cuda")
    state[slots] = dev(S0)
    M = sum(lens)
    y = torch.zeros(M, H * V + 4, dtype=dtype, device="cuda")
    rows = Rows.packed([[0] * n for n in lens], [0] * 4, slots, "cuda")
    head = (inp, ld, *off, a2, rank, b, rank, nw, y, H * V + 4, state)
    tail = (H, D, V, D ** -0.5, 1 / tau, eps, DT[dtype])
    if form == "scan":
        call("llj_gla_scan", *head, rows.row0, rows.slot, 4, *tail)
    else:
        C = _hip.lib().llj_gla_chunk_rows(D, V)
        assert C in (32, 64)
        n, ch, first = rows.chunks(C)
        A, U = torch.empty(M, H * D, device="cuda"), torch.empty(n, H, D, V, device="cuda")
        call("llj_gla_chunks", *head, rows.slot, ch, n, first, 4, A, U, *tail)
    want, S = _gla_ref(off, inp, a2, b, nw, lens, H, D, V, tau, eps, S0)
    close(back(state[slots]), S, 1e-5, "state")
    close(back(y)[:, :H * V], want, 1e-4 if dtype == torch.float32 else 8e-3, "output")
    assert float((state[2] - 9.0).abs().max()) == 0.0


def test_gla_decays_of_any_size(hip):
    """Channels that forget everything at once beside channels that forget nothing, in one chunk: the last token's
    own key must survive, and a marked key 60 tokens back must be seen through the slow channels only."""
    from lit_llama.state import Rows

    g = np.random.default_rng(3)
    H, D, V, rank, n = 1, 32, 32, 4, 200
    bias = np.where(np.arange(D) % 2, 30.0, -80.0)
    off, ld, inp, a2, b, nw = _gla_case(g, [n], H, D, V, rank, torch.float32, bias)
    inp[130, off[1]:off[1] + D] *= 50.0
    rows = Rows.packed([[0] * n], [0], [0], "cuda")
    out = {}
    for form in ("scan", "chunks"):
        state = torch.zeros(1, H, D, V, device="cuda")
        y = torch.zeros(n, V, device="cuda")
        head = (inp, ld, *off, a2, rank, b, rank, nw, y, V, state)
        tail = (H, D, V, D ** -0.5, 4.0, 1e-5, 1)
        if form == "scan":
            call("llj_gla_scan", *head, rows.row0, rows.slot, 1, *tail)
        else:
            k, ch, first = rows.chunks(64)
            A, U = torch.empty(n, D, device="cuda"), torch.empty(k, H, D, V, device="cuda")
            call("llj_gla_chunks", *head, rows.slot, ch, k, first, 1, A, U, *tail)
        out[form] = back(y)
    want, _ = _gla_ref(off, inp, a2, b, nw, [n], H, D, V, 0.25, 1e-5, np.zeros((1, H, D, V)))
    close(out["scan"], want, 1e-4)
    close(out["chunks"], want, 1e-4)


def _latent_case(g, H, D, RD, V, R, n, mark, amp, dtype):
    """Weights and rows of one sequence whose key at `mark` stands out for every query that sees it (a score of
    about amp^2 * scale)."""
    base = 3000.0
    off = [0, (H * (D + RD) + 7) // 8 * 8]
    off.append(off[1] + (H * V + 7) // 8 * 8)
    ld = (off[2] + R + RD + 7) // 8 * 8
    inp = g.standard_normal((n, ld))
    uk, uv = g.standard_normal((H * D, R)) * R ** -0.5, g.standard_normal((H * V, R)) * R ** -0.5
    nw = 1 + 0.2 * g.standard_normal(R)
    # frequencies fall quickly: the last pair hardly turns, so q and k parts along it meet at any distance
    inp[:, off[0]:off[1]][:, [h * (D + RD) + D + RD - 2 for h in range(H)]] = amp
    inp[:, off[2] + R + RD - 2] = 0.0
    inp[mark, off[2] + R + RD - 2] = amp
    return base, off, ld, dev(inp, dtype), dev(uk, dtype), dev(uv, dtype), dev(nw, dtype)


def _latent_ref(inp, off, uk, uv, nw, base, H, D, RD, V, R, win, scale, eps):
    x = back(inp)
    n = len(x)
    c = O.rms(x[:, off[2]:off[2] + R], eps) * back(nw)
    kr = O.rotate_pairs(x[:, off[2] + R:off[2] + R + RD], np.arange(n), base)
    q = x[:, :H * (D + RD)].reshape(n, H, D + RD)
    qr = O.rotate_pairs(q[..., D:], np.arange(n), base)
    ku, v = (c @ back(uk).T).reshape(n, H, D), (c @ back(uv).T).reshape(n, H, V)
    o = np.stack([O.windowed_attention(q[:, h, :D], qr[:, h], ku[:, h], kr, v[:, h], scale, win) for h in range(H)], 1)
    return o.reshape(n, H * V) * O.sigmoid(x[:, off[1]:off[1] + H * V])


@pytest.mark.parametrize("dtype", list(DT))
@pytest.mark.parametrize("H,D,RD,V,R", [(2, 64, 48, 80, 192), (3, 10, 6, 14, 22), (18, 32, 16, 48, 64), (1, 128, 64, 128, 512),
                                        (2, 192, 64, 256, 600)])
@pytest.mark.parametrize("win", [1, 7, 64, 65, 100])
def test_latent_attention(hip, dtype, H, D, RD, V, R, win):
    """Prompt rows in one call, in portions, and as decode rows, with a marked key just inside and just outside of
    the window; a window one key wider or narrower would show far above the tolerance."""
    from lit_llama.mixers import LatentAttention, LatentSpec
    from lit_llama.mugivik import Mugivik  # noqa: F401
    from lit_llama.state import Rows

    n, eps, scale = 150, 1e-5, (D + RD) ** -0.5 * 1.5
    g = np.random.default_rng(win + R)
    base, off, ld, inp, uk, uv, nw = _latent_case(g, H, D, RD, V, R, n, 20, (11.0 / scale) ** 0.5, dtype)
    ref = _latent_ref(inp, off, uk, uv, nw, base, H, D, RD, V, R, win, scale, eps)
    tol = 2e-5 if dtype == torch.float32 else 4e-2
    for d in (-1, 1):
        if win + d > 0:
            other = _latent_ref(inp, off, uk, uv, nw, base, H, D, RD, V, R, win + d, scale, eps)
            assert np.abs(other - ref).max() > 4 * tol * np.abs(ref).max()

    mx = LatentAttention(LatentSpec(H, D, RD, V, R, win, scale, base), 8, eps)
    z = lambda *s: torch.zeros(*s)  # noqa: E731  (projections the test bypasses)
    mx.load({"q": z(H * (D + RD), 8), "g": z(H * V, 8), "dkv": z(R + RD, 8), "o": z(8, H * V), "uk": uk, "uv": uv, "dkv.norm": nw},
            dtype, "cuda")
    assert mx.inp.offset == off

    class Work:
        def __init__(self, x):
            self.proj, self.cur, self.bufs = x, {}, {}

        def buffer(self, name, numel, dt):
            if name not in self.bufs or self.bufs[name].numel() < numel:
                self.bufs[name] = torch.empty(numel, dtype=dt, device="cuda")
            return self.bufs[name]

    class State:
        ring = {0: torch.full((3, win, mx.cache_width(dtype)), 99.0, dtype=dtype, device="cuda")}
        ring_rows = {0: win}

    from lit_llama import _hip

    def prompt(a, b):
        rows = Rows.packed([[0] * (b - a)], [a], [1], "cuda")
        w = Work(inp[a:b].clone())
        y = torch.zeros(b - a, H * V + (-H * V) % 8, dtype=dtype, device="cuda")
        mx.mix(0, rows, w, State, y, _hip.stream())
        mx.commit(0, rows, w, State, _hip.stream())
        return back(y)[:, :H * V]

    def decode(p):
        rows = Rows(1, 1, ints(0), ints(p), ints(1))
        y = torch.zeros(1, H * V, dtype=dtype, device="cuda")
        mx.mix(0, rows, Work(inp[p:p + 1].clone()), State, y, _hip.stream())
        return back(y)

    close(prompt(0, n), ref, tol, "one call")
    got = [prompt(a, min(a + 47, 120)) for a in range(0, 120, 47)] + [decode(p) for p in range(120, n)]
    close(np.concatenate(got), ref, tol, "portions, then decode rows")
    close(np.concatenate([decode(p) for p in range(n)]), ref, tol, "decode rows")


@pytest.mark.parametrize("dtype", list(DT))
def test_next_token_row_positions(hip, dtype):
    g = np.random.default_rng(1)
    lg = dev(g.standard_normal((3, 104)), dtype)
    lg[:, 100:] = 50.0  # columns past the vocabulary
    cur, toks, pos = torch.zeros(3, dtype=torch.int32, device="cuda"), torch.full((3, 9), -1, dtype=torch.int32, device="cuda"), ints(2, 7, 0)
    call("llj_next_token", lg, 104, 3, 100, 1.0, 1, None, 0, cur, toks, 9, pos, 1, DT[dtype])
    want = back(lg)[:, :100].argmax(1)
    assert cur.tolist() == want.tolist()
    exp = np.full((3, 9), -1)
    exp[[0, 1, 2], [3, 8, 1]] = want
    assert (toks.cpu().numpy() == exp).all()
    seen = set()
    for seed in range(40):
        call("llj_next_token", lg, 104, 3, 100, 0.7, 5, None, seed, cur, toks, 9, pos, 1, DT[dtype])
        seen.add(tuple(cur.tolist()))
        for r, t in enumerate(cur.tolist()):
            assert t in np.argsort(-back(lg)[r, :100], kind="stable")[:6]
    assert len(seen) > 10


# ------------------------------------------------------------------------------------ biases and the gated unit
def _unit_ref(y, limit, alpha):
    g, u = np.minimum(y[:, 0::2], limit), np.clip(y[:, 1::2], -limit, limit)
    return g * B.sigmoid(alpha * g) * (u + 1.0)


@pytest.mark.parametrize("M", [1, 8, 9, 16, 64, 100, 256, 300, 1024])
@pytest.mark.parametrize("N,K", [(128, 128), (2048, 1024), (384, 2048), (4352, 1152)])
@pytest.mark.parametrize("act", [0, 2])
def test_bias_and_unit_products(hip, M, N, K, act):
    from lit_llama import _hip

    g = torch.Generator(device="cuda").manual_seed(M + N + K)
    A = torch.randn(M, K, generator=g, device="cuda").to(torch.bfloat16)
    W = (torch.randn(N, K, generator=g, device="cuda") * K ** -0.5).to(torch.bfloat16)
    bias = 2.0 * torch.randn(N, generator=g, device="cuda")
    limit, alpha, C = 1.25, 1.5, N // 2 if act else N
    for b in (bias, None):
        y = back(A) @ back(W).T + (0 if b is None else back(b))
        want = _unit_ref(y, limit, alpha) if act else y
        out = torch.full((M, C + 16), 3.0, dtype=torch.bfloat16, device="cuda")
        if M <= 16:
            call("llj_rows_linear", act, A, K, W, b, out, C + 16, M, N, K, limit, alpha)
            close(back(out)[:, :C], want, 6e-3)
        else:
            nb = _hip.lib().llj_gemm_bf16_ws_bytes(M, N, K)
            for ws in {None, nb or None}:
                buf = None if ws is None else torch.empty(nb // 4, device="cuda")
                out.fill_(3.0)
                call("llj_gemm_bf16", act, A, K, W, b, out, C + 16, M, N, K, limit, alpha, buf, nb)
                close(back(out)[:, :C], want, 6e-3, ws)
        assert float((out[:, C:] - 3.0).abs().max()) == 0.0


@pytest.mark.parametrize("opt", [0, 100])  # LDS-DMA tiles of 256 x 128 / 256 x 256
def test_unit_gemm_tiles(hip, opt):
    from lit_llama import _hip

    g = torch.Generator(device="cuda").manual_seed(opt)
    M, N, K = 520, 512, 256
    A, W = torch.randn(M, K, generator=g, device="cuda").to(torch.bfloat16), (torch.randn(N, K, generator=g, device="cuda") / 16).to(torch.bfloat16)
    bias, y = torch.randn(N, generator=g, device="cuda"), None
    old = _hip.lib().llj_set_option(_hip.OPT_GLDS_COST128, opt)
    try:
        for act, C in ((0, N), (2, N // 2)):
            out = torch.empty(M, C, dtype=torch.bfloat16, device="cuda")
            call("llj_gemm_bf16", act, A, K, W, bias, out, C, M, N, K, 1.0, 1.7, None, 0)
            y = back(A) @ back(W).T + back(bias)
            close(back(out), _unit_ref(y, 1.0, 1.7) if act else y, 6e-3, act)
    finally:
        _hip.lib().llj_set_option(_hip.OPT_GLDS_COST128, old)


@pytest.mark.parametrize("dtype", list(DT))
def test_bias_act(hip, dtype):
    g = np.random.default_rng(3)
    M, N, ld = 5, 42, 48
    y, bias = dev(4 * g.standard_normal((M, ld)), dtype), dev(g.standard_normal(N))
    rel = 2e-6 if dtype == torch.float32 else 6e-3
    out = torch.full((M, 24), 3.0, dtype=dtype, device="cuda")
    for b in (bias, None):
        call("llj_g_bias_act", 2, y, ld, b, out, 24, M, N, 1.5, 1.7, DT[dtype])
        close(back(out)[:, :21], _unit_ref(back(y)[:, :N] + (0 if b is None else back(b)), 1.5, 1.7), rel)
    y0 = back(y)
    call("llj_g_bias_act", 0, y, ld, bias, None, 0, M, N, 0.0, 0.0, DT[dtype])
    close(back(y)[:, :N], y0[:, :N] + back(bias), rel)
    assert (back(y)[:, N:] == y0[:, N:]).all() and float((out[:, 21:] - 3.0).abs().max()) == 0.0


# ------------------------------------------------------------------------------------ residual streams
def _streams_case(g, M, S, C, ld, dtype):
    hc = {"in": dev(g.standard_normal(S)), "out": dev(g.standard_normal(S)), "mix": dev(g.standard_normal((S, S)))}
    x, y = dev(3 + g.standard_normal((M, S, ld))), dev(2 * g.standard_normal((M, ld)), dtype)
    return hc, {k: back(v) for k, v in hc.items()}, x, y, dev(1 + 0.3 * g.standard_normal(C), dtype)


@pytest.mark.parametrize("dtype", list(DT))
@pytest.mark.parametrize("M", [3, 70])
@pytest.mark.parametrize("S,C", [(1, 8), (2, 72), (3, 75), (4, 2048), (3, 4096), (5, 320), (4, 5120), (2, 8192), (2, 9000), (9, 64)])
def test_streams_step(hip, dtype, M, S, C):
    g = np.random.default_rng(C + S)
    ld, eps = (C + 7) // 8 * 8 + 8, 1e-5
    hc, ref, x, y, w = _streams_case(g, M, S, C, ld, dtype)
    X = back(x)[..., :C].transpose(1, 0, 2)
    new = B.streams_out(X, back(y)[:, :C], ref)
    rel = 3e-6 if dtype == torch.float32 else 6e-3
    x0 = x.clone()
    pick = ints(2, 0)
    h = torch.full((M, ld), 7.0, dtype=dtype, device="cuda")
    call("llj_streams_step", y, ld, hc["out"], hc["mix"], x, ld, S, None, w, eps, h, ld, pick, 2, C, DT[dtype])
    assert torch.equal(x, x0)
    close(back(h)[:2, :C], B.layer_norm(new.sum(0), back(w), eps)[[2, 0]], rel, "gathered sum")
    call("llj_streams_step", y, ld, hc["out"], hc["mix"], x, ld, S, hc["in"], w, eps, h, ld, None, M, C, DT[dtype])
    close(back(x)[..., :C].transpose(1, 0, 2), new, 2e-6, "streams")
    close(back(h)[:, :C], B.layer_norm(B.streams_in(new, ref), back(w), eps), rel, "normed")
    assert float(h[:, C:].abs().max()) == 0.0 and torch.equal(x[..., C:], x0[..., C:])


@pytest.mark.parametrize("dtype", list(DT))
@pytest.mark.parametrize("S,C", [(2, 72), (3, 75), (4, 2048), (7, 40)])
def test_streams_embed(hip, dtype, S, C):
    g = np.random.default_rng(S)
    emb, tok = dev(g.standard_normal((11, C)), dtype), ints(3, 10, 0, 3)
    hc, ref, x, _, w = _streams_case(g, 4, S, C, C, dtype)
    h, pos = torch.empty(4, C, dtype=dtype, device="cuda"), ints(5, 0, 2, 9)
    e = back(emb)[[3, 10, 0, 3]] * 1.5
    for ps in (pos, None):
        call("llj_streams_embed", tok, emb, C, 1.5, ps, x, C, S, hc["in"], w, 1e-6, h, C, 4, C, DT[dtype])
        close(back(x), np.stack([e] * S, 1), 1e-6)
        close(back(h), B.layer_norm(ref["in"].sum() * e, back(w), 1e-6), 1e-5 if dtype == torch.float32 else 6e-3)
    assert pos.tolist() == [6, 1, 3, 10]


@pytest.mark.parametrize("S,C,K,N", [(1, 72, 128, 256), (2, 2048, 2048, 384), (4, 4096, 4096, 128), (3, 8192, 8192, 4224),
                                     (4, 1000, 1024, 8448)])
@pytest.mark.parametrize("act", [0, 2])
def test_streams_linear(hip, S, C, K, N, act):
    g = np.random.default_rng(C + N)
    hc, ref, x, y, w = _streams_case(g, 1, S, C, C, torch.bfloat16)
    W, bias = dev(g.standard_normal((N, K)) * C ** -0.5, torch.bfloat16), dev(g.standard_normal(N))
    xo, out = torch.zeros_like(x), torch.empty(N // 2 if act else N, dtype=torch.bfloat16, device="cuda")
    call("llj_streams_linear", act, y, hc["out"], hc["mix"], x, xo, C, S, hc["in"], w, 1e-5, C, W, bias, out, N, K, 1.25, 1.5)
    new = B.streams_out(back(x).transpose(1, 0, 2), back(y), ref)
    close(back(xo).transpose(1, 0, 2), new, 2e-6)
    v = B.layer_norm(B.streams_in(new, ref), back(w), 1e-5) @ back(W)[:, :C].T + back(bias)
    close(back(out), _unit_ref(v, 1.25, 1.5)[0] if act else v[0], 1.2e-2)


# ------------------------------------------------------------------------------------ grouped-query attention
class GqaCase:
    """Packed projections of sequences that go on from `starts` cached tokens, and the float64 reference."""

    def __init__(self, seed, H, G, D, V, RD, starts, lens, dtype, norm=1, sink=1, scale=None, vmode=0, gate=True, plant=None):
        g = np.random.default_rng(seed)
        self.H, self.G, self.D, self.V, self.RD, self.dtype, self.norm, self.sink = H, G, D, V, RD, dtype, norm, sink
        self.starts, self.lens, self.M, self.vmode = starts, lens, sum(lens), vmode
        self.scale = D ** -0.5 if scale is None else scale
        up = lambda n: (n + 7) // 8 * 8  # noqa: E731
        self.o = [0, up(H * D), up(H * D) + up(G * D), up(H * D) + up(G * D) + up(G * V)]
        self.ld, self.W, self.ldc = up(self.o[3] + H), max(a + b for a, b in zip(starts, lens)) + 3, up(G * (D + V))
        self.eps, self.base, self.factor = 1e-5, 70.0, 1.5
        self.inp = dev(1.5 * g.standard_normal((self.M, self.ld)), dtype)
        self.slots = list(g.permutation(len(lens) + 2)[:len(lens)])
        self.cache = dev(g.standard_normal((len(lens) + 2, self.W, self.ldc)), dtype)
        if plant is not None:  # every query and one key per sequence share a direction
            q, c = back(self.inp), back(self.cache)
            q[:, :H * D].reshape(self.M, H, D)[:, :, -1] = 6.0
            q[:, self.o[1]:self.o[1] + G * D].reshape(self.M, G, D)[:, :, -1] = 0.0
            c[:, :, :G * D].reshape(-1, self.W, G, D)[..., -1] = 0.0
            row = 0
            for s, n, sl in zip(starts, lens, self.slots):
                if plant < s:
                    c[sl, plant, :G * D].reshape(G, D)[:, -1] = 6.0
                elif plant < s + n:
                    q[row + plant - s, self.o[1]:self.o[1] + G * D].reshape(G, D)[:, -1] = 6.0
                row += n
            self.inp, self.cache = dev(q, dtype), dev(c, dtype)
        self.lam, self.first = dev([0.3]), dev(g.standard_normal((self.M, G * V)), dtype)
        self.gate = gate
        i = torch.arange(0, RD, 2, dtype=torch.float64)
        self.turns = (self.base ** (-i / max(RD, 1)) / self.factor / (2 * np.pi)).cuda()
        self.pos = ints(*[s + j for s, n in zip(starts, lens) for j in range(n)])
        self.seq = ints(*[b for b, n in enumerate(lens) for _ in range(n)])
        self.slot = ints(*self.slots)
        self.args = (self.M, H, G, D, V)

    def reference(self):
        """(outputs, cache after, first after)"""
        H, G, D, V, o = self.H, self.G, self.D, self.V, self.o
        p, cache, first = back(self.inp), back(self.cache), back(self.first)
        pos = np.array(self.pos.tolist())
        def prep(t):
            t = B.rotate_half(t, pos, self.base, self.RD, self.factor) if self.RD else t
            return B.unit_rms(t, self.eps) if self.norm else t
        q, k = prep(p[:, :H * D].reshape(-1, H, D)), prep(p[:, o[1]:o[1] + G * D].reshape(-1, G, D))
        v = p[:, o[2]:o[2] + G * V]
        if self.vmode == 1:
            first = v.copy()
        elif self.vmode == 2:
            v = B.mix_values(v, first, float(back(self.lam)[0]))
        y, row = np.empty((self.M, H * V)), 0
        for s, n, sl in zip(self.starts, self.lens, self.slots):
            r = slice(row, row + n)
            cache[sl, s:s + n, :G * D], cache[sl, s:s + n, G * D:G * (D + V)] = k[r].reshape(n, -1), v[r]
            K, Vv = cache[sl, :s + n, :G * D].reshape(-1, G, D), cache[sl, :s + n, G * D:G * (D + V)].reshape(-1, G, V)
            for i in range(n):
                for h in range(H):
                    gh, e = h // (H // G), s + i + 1
                    sc = K[:e, gh] @ q[row + i, h] * self.scale
                    m = max(sc.max(), 0.0) if self.sink else sc.max()
                    w = np.exp(sc - m)
                    out = w @ Vv[:e, gh] / (w.sum() + (np.exp(-m) if self.sink else 0.0))
                    y[row + i, h * V:(h + 1) * V] = out * (B.sigmoid(p[row + i, o[3] + h]) if self.gate else 1.0)
            row += n
        return y, cache, first

    def new(self):
        """arguments for the rows' own keys and values"""
        first = self.first if self.vmode else None
        return (self.pos,), (self.turns, self.RD, self.norm, self.eps), (first, self.lam if self.vmode == 2 else None, self.G * self.V)

    def og(self):
        return self.o[3] if self.gate else -1

    def verify(self, y, what=""):
        want, cache, first = self.want
        f32 = self.dtype == torch.float32
        close(back(y)[:, :self.H * self.V], want, 5e-6 if f32 else 2e-2, what)
        n = self.G * (self.D + self.V)
        close(back(self.cache)[..., :n], cache[..., :n], 3e-6 if f32 else 8e-3, f"{what} cache")
        close(back(self.first), first, 1e-7, f"{what} first values")

    def run(self, kind):
        self.want = self.reference()
        y = torch.zeros(self.M, (self.H * self.V + 7) // 8 * 8, dtype=self.dtype, device="cuda")
        o, dt = self.o, DT[self.dtype]
        (pos,), rot, mixed = self.new()
        if kind == "decode":
            from lit_llama import _hip

            count = torch.zeros(self.M * self.H, dtype=torch.int32, device="cuda")
            for n in (1, 2, 7, 16):
                part = torch.full((self.M * self.H * n * _hip.lib().llj_gqa_part_width(self.V),), 9.0, device="cuda")
                call("llj_gqa_decode", self.inp, self.ld, *o[:3], self.og(), *rot, pos, self.slot, self.cache, self.W, self.ldc,
                     *mixed, part, count, n, y, y.stride(0), *self.args, self.scale, self.sink)
                self.verify(y, n)
                assert int(count.abs().max()) == 0
            return
        call("llj_gqa_prep", self.inp, self.ld, *o[:3], *rot, pos, self.seq, self.slot, self.cache, self.W, self.ldc, *mixed,
             *self.args, dt)
        if kind == "rows":
            call("llj_gqa_rows", self.inp, self.ld, o[0], self.og(), pos, self.seq, self.slot, self.cache, self.W, self.ldc, y,
                 y.stride(0), *self.args, self.scale, self.sink, dt)
        else:
            from lit_llama.state import Rows

            r = Rows.packed([[0] * n for n in self.lens], self.starts, [int(s) for s in self.slots], "cuda")
            n, work = r.pairs(kind)
            call("llj_gqa_flash", self.inp, self.ld, o[0], self.og(), work, n, kind, pos, self.slot, self.cache, self.W, self.ldc, y,
                 y.stride(0), *self.args, self.scale, self.sink)
        self.verify(y, kind)


GQA_SIZES = [(3, 1, 10, 14, 6), (4, 2, 7, 5, 0), (2, 2, 1, 1, 0), (6, 2, 48, 24, 16), (8, 1, 128, 128, 128), (20, 1, 96, 64, 64),
             (2, 1, 256, 168, 32), (40, 2, 64, 96, 64), (1, 1, 600, 300, 320)]


@pytest.mark.parametrize("dtype", list(DT))
@pytest.mark.parametrize("H,G,D,V,RD", GQA_SIZES)
@pytest.mark.parametrize("vmode", [0, 1, 2])
def test_gqa_rows(hip, dtype, H, G, D, V, RD, vmode):
    GqaCase(D + vmode, H, G, D, V, RD, [0, 40, 300], [5, 1, 3], dtype, vmode=vmode).run("rows")


@pytest.mark.parametrize("H,G,D,V,RD", [s for s in GQA_SIZES if s[2] % 8 == 0 and s[3] % 8 == 0 and s[2] <= 256])
@pytest.mark.parametrize("rows", [64, 128])
def test_gqa_flash(hip, H, G, D, V, RD, rows):
    if rows == 128 and max(D, V) > 128:
        pytest.skip("64-query blocks only")
    GqaCase(D, H, G, D, V, RD, [0, 40, 0], [70, 130, 200], torch.bfloat16, vmode=2).run(rows)


@pytest.mark.parametrize("H,G,D,V,RD", [s for s in GQA_SIZES if s[2] % 8 == 0 and s[3] % 8 == 0 and s[2] <= 256])
@pytest.mark.parametrize("vmode", [0, 1, 2])
def test_gqa_decode(hip, H, G, D, V, RD, vmode):
    GqaCase(D + vmode, H, G, D, V, RD, [0, 1, 31, 32, 33, 127, 128, 500], [1] * 8, torch.bfloat16, vmode=vmode).run("decode")


@pytest.mark.parametrize("kind,dtype", [("rows", torch.float32), ("rows", torch.bfloat16), (64, torch.bfloat16), (128, torch.bfloat16),
                                        ("decode", torch.bfloat16)])
@pytest.mark.parametrize("option", [dict(norm=0), dict(sink=0), dict(gate=False), dict(norm=0, scale=-0.2), dict(scale=1.5),
                                    dict(norm=0, scale=0.6), dict(norm=0, scale=0.6, sink=0)])
def test_gqa_options(hip, kind, dtype, option):
    lens = [1] * 3 if kind == "decode" else [66, 3, 90]
    GqaCase(5, 6, 2, 48, 24, 32, [0, 90, 33], lens, dtype, **option).run(kind)


@pytest.mark.parametrize("kind,dtype", [("rows", torch.float32), (64, torch.bfloat16), (128, torch.bfloat16), ("decode", torch.bfloat16)])
@pytest.mark.parametrize("key", [0, 1, 15, 16, 31, 32, 63, 64, 95, 96, 127, 128, 199, 200])
def test_gqa_one_key_stands_out(hip, kind, dtype, key):
    """Each query's weight lies almost wholly on one key (its own, or one at a tile's edge): the output is that value."""
    starts, lens = ([200, key, 230], [1, 1, 1]) if kind == "decode" else ([0, key, 100], [202, 4, 105])
    c = GqaCase(key, 4, 2, 32, 16, 16, starts, lens, dtype, norm=0, scale=0.5, plant=key)
    c.run(kind)


@pytest.mark.parametrize("kind,dtype", [("rows", torch.float32), (64, torch.bfloat16), ("decode", torch.bfloat16)])
def test_gqa_sink_takes_the_weight(hip, kind, dtype):
    """Scores far below 0 leave the weight to the sink: the outputs almost vanish, and would be averages without it."""
    lens = [1] * 2 if kind == "decode" else [70, 9]
    c = GqaCase(1, 2, 1, 32, 16, 0, [0, 64], lens, dtype, norm=0, scale=1.0, gate=False)
    q, k = back(c.inp), back(c.cache)
    q[:, :64] = 1.0
    q[:, c.o[1]:c.o[1] + 32] = -0.2
    k[..., :32] = -0.2
    c.inp, c.cache = dev(q, dtype), dev(k, dtype)
    c.run(kind)
    assert np.abs(c.want[0]).max() < 0.15
