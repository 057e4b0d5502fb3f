"""numpy restatement of the Bobasun decoder — TEST INFRASTRUCTURE (see oracle/__init__.py).

A decoder whose residual is several streams, mixed by small learned matrices around every sublayer;
grouped-query attention with normalized rotated queries and keys, a sink of score 0, values mixed with the
first mixing layer's and one output gate per head; feed-forwards with a clamped gated activation; biased
projections, bias-free layer norms on the sublayers' inputs, an untied head.

One function per mechanism, a sequence recomputed from its first token without caches. Computes in `F`
(float64 by default, so that the float32 product path is compared with something more exact than
itself). `params` maps tensor names to arrays; `cfg` is the plain dict of config.json.
"""
from __future__ import annotations

import numpy as np

F = np.float64


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdims=True)
    return d / np.sqrt((d * d).mean(-1, keepdims=True) + eps) * w


def unit_rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def sigmoid(z):
    return np.exp(-np.logaddexp(0.0, -z))


def linear(h, P, name):
    """W h, plus the bias where the checkpoint has one."""
    y = h @ P[name].T
    return y + P[name + ".b"] if name + ".b" in P else y


def rotate_half(x, positions, base, dims, factor):
    """Rotary positions on the first `dims` of the last axis, dimension i with dimension i + dims / 2;
    frequencies base^(-2 i / dims) / factor; x (T, heads, dim)."""
    n = dims // 2
    f = base ** (-2.0 * np.arange(n) / dims) / factor
    a = np.asarray(positions, F)[:, None, None] * f
    c, s = np.cos(a), np.sin(a)
    out = x.copy()
    u, v = x[..., :n], x[..., n:dims]
    out[..., :n] = u * c - v * s
    out[..., n:dims] = v * c + u * s
    return out


def sink_attention(q, k, v, scale):
    """One head, causal: weights exp(s_j) / (1 + sum exp(s)); q, k (T, dim), v (T, vdim)."""
    out = np.empty((q.shape[0], v.shape[1]), q.dtype)
    for i in range(q.shape[0]):
        s = k[:i + 1] @ q[i] * scale
        m = max(0.0, s.max())
        e = np.exp(s - m)
        out[i] = (e / (np.exp(-m) + e.sum())) @ v[:i + 1]
    return out


def mix_values(v, first, lam):
    return (1.0 - lam) * v + lam * first


def attention(h, m, P, pre, eps, first):
    """Attention over a whole sequence; h (T, width). `first`: the values of the first mixing layer, None in
    that layer itself and in layers that do not mix. Returns (output, this layer's own values)."""
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T, rot = h.shape[0], m["rot"]
    pos = np.arange(T)
    q = linear(h, P, pre + "q").reshape(T, H, D)
    k = linear(h, P, pre + "k").reshape(T, G, D)
    v = linear(h, P, pre + "v").reshape(T, G, V)
    q, k = (unit_rms(rotate_half(t, pos, rot["base"], rot["dims"], rot["scaling"]["factor"]), eps) for t in (q, k))
    own = v
    if first is not None:
        v = mix_values(v, first, float(P[pre + "vmix"]))
    gate = sigmoid(h @ P[pre + "g"].T)
    o = np.empty((T, H, V), h.dtype)
    for i in range(H):
        g = i // (H // G)
        o[:, i] = sink_attention(q[:, i], k[:, g], v[:, g], m["scale"]) * gate[:, i:i + 1]
    return linear(o.reshape(T, H * V), P, pre + "o"), own


def clamped_glu(g, u, limit):
    g, u = np.minimum(g, limit), np.clip(u, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


def feed_forward(h, f, P, pre):
    return linear(clamped_glu(linear(h, P, pre + "gate"), linear(h, P, pre + "up"), f["limit"]), P, pre + "down")


def streams_in(X, hc):
    """A sublayer's input from the streams X (S, T, width)."""
    return np.einsum("s,stc->tc", hc["in"], X)


def streams_out(X, y, hc):
    """The streams after a sublayer: from s to t by mix[s, t], its output y by out[t]."""
    return np.einsum("sr,stc->rtc", hc["mix"], X) + hc["out"][:, None, None] * y


def forward(tokens, cfg, params, layers_out=None):
    """Logits (T, vocab) of one sequence; layers_out, a list, receives the sum of the streams after every layer."""
    P = {k: np.asarray(a, F) for k, a in params.items()}
    eps = cfg["norm"]["eps"]
    x = P["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    X = np.stack([x] * cfg["streams"])
    first = None
    for i, L in enumerate(cfg["layers"]):
        pre = f"l{i}."
        hc = {n: P[f"{pre}hc1.{n}"] for n in ("in", "out", "mix")}
        mixes = bool(L["mixer"].get("v_mix"))
        y, own = attention(layer_norm(streams_in(X, hc), P[pre + "norm1"], eps), L["mixer"], P, pre + "mix.", eps,
                           first if mixes else None)
        if mixes and first is None:
            first = own
        X = streams_out(X, y, hc)
        if L.get("mlp") is not None:
            hc = {n: P[f"{pre}hc2.{n}"] for n in ("in", "out", "mix")}
            y = feed_forward(layer_norm(streams_in(X, hc), P[pre + "norm2"], eps), L["mlp"], P, pre + "mlp.")
            X = streams_out(X, y, hc)
        if layers_out is not None:
            layers_out.append(X.sum(0))
    return layer_norm(X.sum(0), P["final.norm"], eps) @ P["head"].T
