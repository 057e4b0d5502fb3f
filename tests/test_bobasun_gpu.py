"""Bobasun on the device against oracle/bobasun_np.py (float64, recomputed from the first token): whole prompts, token
by token, portions, batches of unequal requests, slots used again, far keys and tile borders, the first tokens, long
decoding past grown caches, greedy generation. Tolerances as for the other models with per-sequence state."""
import copy

import numpy as np
import pytest
import torch

from oracle import bobasun_np as O
from tests.bobasun_cases import CONFIGS, TOL, build, check, config, errors, layer, oracle, prompts, weights

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
_cache = {}


def case(name, dtype, seed=0):
    key = (name, dtype, seed)
    if key not in _cache:
        cfg = CONFIGS[name]
        w = weights(cfg, seed)
        _cache[key] = (cfg, w, build(cfg, w, dtype))
    return _cache[key]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompts(hip, name, dtype):
    cfg, w, m = case(name, dtype)
    for n in (1, 2, 3, 17, 64, 65, 150, 300):
        toks = prompts(cfg, [n], seed=n)[0]
        st = m.new_state(1)
        got = m.extend(st, st.alloc(1), [0], [toks])
        check(got, oracle(cfg, w, toks), dtype, (name, n))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("wide", [1, 256])
def test_long_prompt(hip, monkeypatch, dtype, wide):
    """Long prompts in both query block sizes, several tiles of keys and the split products."""
    from lit_llama import mixers

    monkeypatch.setattr(mixers, "GQA_WIDE_WGS", wide)
    cfg, w, m = case("tiled", dtype)
    toks = prompts(cfg, [1100], seed=21)[0]
    st = m.new_state(1)
    check(m.extend(st, st.alloc(1), [0], [toks]), oracle(cfg, w, toks), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_streams_after_every_layer(hip, name, dtype):
    cfg, w, m = case(name, dtype)
    for n in (1, 90):
        toks = prompts(cfg, [n], seed=5)[0]
        taps, want = [], []
        st = m.new_state(1)
        got = m.extend(st, st.alloc(1), [0], [toks], taps=taps)
        ref = O.forward(toks, cfg, w, want)
        assert len(taps) == len(want) == len(cfg["layers"])
        for i, (a, b) in enumerate(zip(taps, want)):
            assert np.abs(a.cpu().numpy() - b).max() < (5e-5 if dtype == torch.float32 else 0.1) * np.abs(b).max(), i
        check(got, ref, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_token_by_token_equals_prompt(hip, name, dtype):
    """Decode steps (the session's captured graph) from the first token on, past tiles of keys."""
    from lit_llama.engine import DecodeSession

    cfg, w, m = case(name, dtype)
    toks = prompts(cfg, [160], seed=2)[0]
    ref = oracle(cfg, w, toks)
    s = DecodeSession(m, 1, None, None, keep_tokens=False)
    out = [s.prefill([toks[:1]], want=[[0]]).clone()]
    for t in toks[1:]:
        out.append(s.feed([t]).clone())
    check(torch.cat(out), ref, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["odd", "tiled", "wide"])
@pytest.mark.parametrize("portion", [2, 7, 64, 100])
def test_portions(hip, name, dtype, portion):
    cfg, w, m = case(name, dtype)
    toks = prompts(cfg, [40 if portion == 2 else 210], seed=3)[0]
    ref = oracle(cfg, w, toks)
    st = m.new_state(1)
    slot = st.alloc(1)
    got = [m.extend(st, slot, [p], [toks[p:p + portion]]) for p in range(0, len(toks), portion)]
    check(torch.cat(got), ref, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["odd", "tiled", "wide"])
def test_unequal_batch_and_early_ends(hip, name, dtype):
    """Prompts of different lengths in one call, decoded together, ending one by one; the freed slots, still full of
    the old rows, serve a second batch."""
    from lit_llama.engine import DecodeSession

    cfg, w, m = case(name, dtype)
    state = m.new_state(4)
    for turn in range(2):
        lens = [1, 150, 37, 70] if turn == 0 else [66, 2, 129]
        extra = [3, 9, 6, 9] if turn == 0 else [5, 12, 1]
        toks = prompts(cfg, [a + b for a, b in zip(lens, extra)], seed=10 + turn)
        refs = [oracle(cfg, w, t) for t in toks]
        s = DecodeSession(m, len(lens), None, None, state=state, keep_tokens=False)
        want = [sorted({0, n // 2, n - 1}) for n in lens]
        got = s.prefill([t[:n] for t, n in zip(toks, lens)], want=want)
        check(got, np.concatenate([r[k] for r, k in zip(refs, want)]), dtype)
        live, at, outs, wants = list(range(len(lens))), list(lens), [], []
        while live:
            outs.append(s.feed([toks[i][at[i]] for i in live]).clone())
            wants += [refs[i][at[i]] for i in live]
            for i in live:
                at[i] += 1
            done = [k for k, i in enumerate(live) if at[i] == len(toks[i])]
            if done:
                s.finish(done)
                live = [i for k, i in enumerate(live) if k not in done]
        check(torch.cat(outs), np.stack(wants), dtype)
        assert len(state._free) == 4


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("batch", [2, 5, 8, 11, 19, 70])
def test_batched_decode_rows(hip, dtype, batch):
    """Every batch size class of the decode kernels: rows equal their own sequences."""
    from lit_llama.engine import DecodeSession

    cfg, w, m = case("tiled", dtype)
    toks = prompts(cfg, [30 + (7 * b) % 11 for b in range(batch)], seed=batch)
    s = DecodeSession(m, batch, None, None, keep_tokens=False)
    s.prefill([t[:-3] for t in toks])
    for k in (3, 2, 1):
        out = s.feed([t[-k] for t in toks])
        want = np.stack([oracle(cfg, w, t[:len(t) - k + 1])[-1] for t in toks])
        check(out, want, dtype, k)


def _attention_without(drop=None, sink=True):
    """The oracle's attention with a key left out (for the queries after it) or without the sink."""
    def f(q, k, v, scale):
        out = np.empty((q.shape[0], v.shape[1]))
        for i in range(q.shape[0]):
            keep = [j for j in range(i + 1) if j != drop or j == i]
            s = k[keep] @ q[i] * scale
            m = max(0.0, s.max())
            e = np.exp(s - m)
            out[i] = (e / ((np.exp(-m) if sink else 0.0) + e.sum())) @ v[keep]
        return out

    return f


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("key", [0, 1, 31, 32, 63, 64, 127, 128, 200])
def test_far_keys_and_tile_borders_show(hip, monkeypatch, dtype, key):
    """One token's keys stand out (a large component that the position leaves alone): leaving that single key out would
    show far above the tolerance at every later position, in prompts and in decoding."""
    from lit_llama.engine import DecodeSession

    cfg = config(64, 50, 2, [layer(4, 2, 32, 24, 64, 8, scale=0.4)] * 2)
    w = dict(weights(cfg, 7))
    # token 49: direction 5 of the width; every query looks for it, its keys answer
    w["embed"] = w["embed"].copy()
    w["embed"][:, 5] = 0.0
    w["embed"][49] = 0.0
    w["embed"][49, 5] = 6.0
    for i in range(2):
        b = np.zeros(4 * 32, np.float32)
        b[31::32] = 4.0
        w[f"l{i}.mix.q.b"] = b
        k = w[f"l{i}.mix.k"].copy()
        k[31::32] = 0.0
        k[31::32, 5] = 4.0
        w[f"l{i}.mix.k"] = k
    m = build(cfg, w, dtype)
    toks = [t % 49 for t in prompts(cfg, [230], seed=6)[0]]
    toks[key] = 49
    ref = oracle(cfg, w, toks)
    with monkeypatch.context() as mp:
        mp.setattr(O, "sink_attention", _attention_without(key))
        e = errors(oracle(cfg, w, toks)[key + 1:], ref[key + 1:])
        assert e[0] > 2 * TOL[dtype][0], e
    st = m.new_state(1)
    check(m.extend(st, st.alloc(1), [0], [toks])[key + 1:], ref[key + 1:], dtype)
    s = DecodeSession(m, 1, None, None, keep_tokens=False)
    s.prefill([toks[:10]])
    out = torch.stack([s.feed([t])[0].clone() for t in toks[10:]])
    check(out[max(0, key - 9):], ref[max(10, key + 1):], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_sink_shows_at_the_first_tokens(hip, monkeypatch, dtype):
    """The sink weighs most where few keys are seen: without it the first rows would be far off."""
    cfg, w, m = case("tiled", dtype)
    toks = prompts(cfg, [4, 1, 3], seed=8)
    refs = [oracle(cfg, w, t) for t in toks]
    with monkeypatch.context() as mp:
        mp.setattr(O, "sink_attention", _attention_without(sink=False))
        for t, r in zip(toks, refs):
            assert errors(oracle(cfg, w, t), r)[0] > 3 * TOL[dtype][0]
    st = m.new_state(3)
    slots = st.alloc(3)
    check(m.extend(st, slots, [0, 0, 0], toks), np.concatenate(refs), dtype)
    st.release(slots[1:2])  # a slot used again starts like new
    again = st.alloc(1)
    assert again == slots[1:2]
    check(m.extend(st, again, [0], [toks[2]]), refs[2], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(hip, dtype):
    """Hundreds of decoded tokens: the cache grows under the captured step, which is captured again."""
    from lit_llama.engine import DecodeSession

    cfg, w, m = case("odd", dtype)
    toks = prompts(cfg, [700], seed=9)[0]
    ref = oracle(cfg, w, toks)
    s = DecodeSession(m, 1, None, None, keep_tokens=False)
    s.prefill([toks[:50]])
    assert s.program.state.ring_rows[0] == 256
    out = torch.stack([s.feed([t])[0].clone() for t in toks[50:]])
    assert s.program.state.ring_rows[0] == 1024
    check(out, ref[50:], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_split_decode_at_every_length(hip, dtype):
    """A wide cache splits the keys over many workgroups: short sequences leave most of them empty."""
    from lit_llama.engine import DecodeSession

    cfg, w, m = case("many", dtype)
    toks = prompts(cfg, [300, 300], seed=14)
    refs = [oracle(cfg, w, t) for t in toks]
    s = DecodeSession(m, 2, 4096, None, keep_tokens=False)
    s.prefill([toks[0][:1], toks[1][:30]])
    outs, wants = [], []
    for k in range(270):
        outs.append(s.feed([toks[0][1 + k], toks[1][30 + k]]).clone())
        wants += [refs[0][1 + k], refs[1][30 + k]]
    check(torch.cat(outs), np.stack(wants), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_large_inputs_of_the_unit(hip, dtype):
    """Gates and ups far past the limit on both sides, in prompt and decode products."""
    cfg = config(128, 60, 3, [layer(2, 1, 16, 16, 200, limit=1.5), layer(2, 1, 16, 16, 200, limit=0.25)])
    w = {k: v * 8.0 if k.endswith((".gate", ".up")) else v for k, v in weights(cfg, 2).items()}
    m = build(cfg, w, dtype)
    toks = prompts(cfg, [90], seed=4)[0]
    ref = oracle(cfg, w, toks)
    st = m.new_state(1)
    slot = st.alloc(1)
    got = m.extend(st, slot, [0], [toks[:70]])
    check(torch.cat([got] + [m.extend(st, slot, [p], [toks[p:p + 10]]) for p in (70, 80)]), ref, dtype)


def test_greedy_generation_float32(hip):
    """generate() and generate_batch() on unequal prompts go through the framework's own loop; greedy ids equal the
    oracle's."""
    import generate as G

    cfg, w, m = case("tiled", torch.float32)
    toks = prompts(cfg, [23, 5, 61], seed=12)
    want = []
    for t in toks:
        t = list(t)
        for _ in range(12):
            t.append(int(oracle(cfg, w, t)[-1].argmax()))
        want.append(t)
    for t, r in zip(toks, want):
        got = G.generate(m, torch.tensor(t).cuda(), 12, top_k=1)
        assert got.tolist() == r
    rows = G.generate_batch(m, [torch.tensor(t) for t in toks], 12)
    assert [r.tolist() for r in rows] == want
    torch.manual_seed(3)
    a = G.generate(m, torch.tensor(toks[1]).cuda(), 20, top_k=7, temperature=0.9)
    torch.manual_seed(3)
    b = G.generate(m, torch.tensor(toks[1]).cuda(), 20, top_k=7, temperature=0.9)
    assert a.tolist() == b.tolist() and max(a.tolist()) < cfg["vocab"]


@pytest.mark.parametrize("name,batch", [("wide", 1), ("wide", 2), ("tiled", 3)])
def test_graph_replays_equal_eager_steps(hip, name, batch):
    """Replays of the captured step, with eager work in between, give the eager steps' ids."""
    from lit_llama.engine import DecodeSession

    cfg, w, m = case(name, torch.bfloat16)
    toks = prompts(cfg, [20, 33, 7][:batch], seed=13)
    runs = []
    for graph in (True, False):
        s = DecodeSession(m, batch, 200, 200, use_graph=graph)
        s.prefill(toks)
        for n in (1, 5, 2, 40):
            s.decode(n)
            torch.cuda.synchronize()
            torch.ones(1000, device="cuda").sum().item()
        runs.append([r.tolist() for r in s.output()])
    assert runs[0] == runs[1]


def test_model_folder_forward_cli_and_replay(hip, tmp_path, capsys, monkeypatch):
    """A folder (config.json + model.safetensors) through load_model, LLaMA-style forward, generate.py and the trace
    replay."""
    import io
    import json

    import generate as G
    from lit_llama import load_model, trace
    from safetensors.torch import save_file

    cfg, w, m = case("odd", torch.float32)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: torch.from_numpy(np.array(v)).to(torch.bfloat16).contiguous() for k, v in w.items()},
              str(tmp_path / "model.safetensors"))
    f = load_model(tmp_path, torch.float32)
    idx = torch.tensor(prompts(cfg, [30, 30], seed=20)).cuda()
    ref = np.stack([oracle(cfg, w, t) for t in idx.tolist()])
    check(f(idx).reshape(60, -1), ref.reshape(60, -1), torch.float32)
    got = [f(idx[:, :12], 40, torch.arange(12)), f(idx[:, 12:13], 40, torch.tensor([12])), f(idx[:, 13:], 40, torch.arange(13, 30))]
    check(torch.cat(got, 1).reshape(60, -1), ref.reshape(60, -1), torch.float32)
    f.reset_cache()
    G.main(checkpoint_path=tmp_path, prompt_tokens=idx[0].tolist(), max_new_tokens=6, top_k=1, dtype="float32")
    out = [int(x) for x in capsys.readouterr().out.split()]
    assert out == G.generate(m, idx[0], 6, top_k=1).tolist()
    a, b = idx.tolist()
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:9], "want": [0, 8]}, {"id": "b", "tokens": b[:20], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[20:21], "want": [0]}, {"id": "a", "tokens": a[9:10], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[10:11], "want": [0]}], "end": ["a"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
    assert trace.main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path)]) == 0
    assert capsys.readouterr().out.split() == ["done", "0", "done", "1", "done", "2"]
    want = [ref[0][[0, 8]], np.stack([ref[1][20], ref[0][9]]), ref[0][[10]]]
    for i, r in enumerate(want):
        check(np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(len(r), -1), r, torch.float32)


def test_refused_configurations(hip):
    """What no kernel takes is refused on the host."""
    from lit_llama import _hip

    cfg, w, m = case("tiled", torch.float32)
    st = m.new_state(1, 8)
    with pytest.raises(ValueError):
        m.extend(st, st.alloc(1), [0], [list(range(9))])
    c = copy.deepcopy(cfg)
    c["streams"] = 200  # more than a workgroup's LDS holds
    with pytest.raises(_hip.HipError):
        b = build(c, weights(c), torch.float32)
        st = b.new_state(1)
        b.extend(st, st.alloc(1), [0], [[1, 2]])
