"""Mugivik without a GPU: configuration reading, tensor checks, slot bookkeeping, the safetensors reader, and
the oracle's own consistency."""
import copy
import json
import struct

import numpy as np
import pytest
import torch

from oracle import mugivik_np as O
from tests.mugivik_cases import CONFIGS, build, oracle, prompts, weights


def _cfg(d):
    from lit_llama.mugivik import MugivikConfig

    return MugivikConfig.from_dict(d)


@pytest.mark.parametrize("name", list(CONFIGS))
def test_config_and_tensors(name):
    cfg = CONFIGS[name]
    c = _cfg(json.loads(json.dumps(cfg)))
    assert c.n_layer == len(cfg["layers"]) and c.vocab_size == cfg["vocab"]
    w = weights(cfg)
    m = build(cfg, w, torch.float32, "cpu")
    assert m.embed.w.shape[0] >= cfg["vocab"]
    bad = dict(w)
    bad.pop("final.norm")
    with pytest.raises(ValueError, match="final.norm"):
        build(cfg, bad, torch.float32, "cpu")
    with pytest.raises(ValueError, match="unexpected"):
        build(cfg, dict(w, extra=w["embed"]), torch.float32, "cpu")
    with pytest.raises(ValueError, match="shape"):
        build(cfg, dict(w, **{"embed.norm": w["embed.norm"][1:]}), torch.float32, "cpu")


def test_config_errors():
    base = CONFIGS["odd"]

    def broken(edit):
        d = copy.deepcopy(base)
        edit(d)
        with pytest.raises(ValueError):
            from lit_llama.mugivik import Mugivik

            Mugivik(_cfg(d))

    broken(lambda d: d.update(extra=1))
    broken(lambda d: d["layers"][0].update(type="other"))
    broken(lambda d: d["layers"][0]["mixer"]["rot"].update(dims=4))
    broken(lambda d: d["layers"][2]["mixer"].update(kv_from=1))  # a recurrent layer has no latents
    broken(lambda d: d["layers"][2]["mixer"].update(kv_from=3))  # not an earlier layer
    broken(lambda d: d["layers"][2]["mixer"].update(kv_rank=23))  # must agree with its owner
    broken(lambda d: d["layers"][0]["mlp"].update(kind="other"))
    broken(lambda d: d["layers"][0]["mixer"]["mask"].update(size=0))
    broken(lambda d: d["norm"].update(eps2=1))


def test_ring_covers_the_widest_reader():
    from lit_llama.mugivik import Mugivik

    m = Mugivik(_cfg(CONFIGS["odd"]))
    assert m.mixers[0].ring_window() == 11 and m.mixers[2].ring_window() is None
    m = build(CONFIGS["odd"], weights(CONFIGS["odd"]), torch.float32, "cpu")
    assert m.new_state(2).ring_rows == {0: 11}
    assert m.new_state(2, 6).ring_rows == {0: 6}


def test_slots():
    m = build(CONFIGS["odd"], weights(CONFIGS["odd"]), torch.float32, "cpu")
    st = m.new_state(3)
    a = st.alloc(2)
    st.recurrent[1][a[0]] += 1.0
    st.prev[a[0]] = 5
    with pytest.raises(RuntimeError):
        st.alloc(2)
    with pytest.raises(RuntimeError):
        st.reserve(2)  # cannot grow while sequences live
    st.release(a)
    with pytest.raises(ValueError):
        st.release(a[:1])
    b = st.alloc(3)
    assert sorted(b) == [0, 1, 2]
    assert float(st.recurrent[1].abs().max()) == 0.0 and st.prev.tolist() == [-1] * 3
    st.release(b)
    st.reserve(5)
    assert st.slots == 5 and len(st.alloc(5)) == 5


def test_packed_rows():
    from lit_llama.state import Rows

    r = Rows.packed([[4, 5, 6], [7]], [0, 9], [2, 0], "cpu")
    assert r.M == 4 and r.B == 2 and not r.decode
    assert r.tok.tolist() == [4, 5, 6, 7] and r.pos.tolist() == [0, 1, 2, 9] and r.row_seq.tolist() == [0, 0, 0, 1]
    assert r.row0.tolist() == [0, 3, 4] and r.slot.tolist() == [2, 0]
    with pytest.raises(ValueError):
        Rows.packed([[1], []], [0, 0], [0, 1], "cpu")


def test_safetensors_reader(tmp_path):
    from lit_llama.checkpoint import read_safetensors
    from safetensors.torch import save_file

    t = {"a": torch.randn(3, 5).to(torch.bfloat16), "b": torch.arange(7, dtype=torch.int32), "c": torch.randn(2, 2, 2),
         "d": torch.zeros(0, 4)}
    save_file(t, str(tmp_path / "m.safetensors"), metadata={"k": "v"})
    got = read_safetensors(tmp_path / "m.safetensors")
    assert set(got) == set(t) and all(torch.equal(got[k], t[k]) and got[k].dtype == t[k].dtype for k in t)
    head = json.dumps({"a": {"dtype": "F32", "shape": [4], "data_offsets": [0, 16]}}).encode()
    (tmp_path / "short").write_bytes(struct.pack("<Q", len(head)) + head + b"\0" * 8)
    with pytest.raises(ValueError):
        read_safetensors(tmp_path / "short")
    (tmp_path / "junk").write_bytes(b"\xff" * 40)
    with pytest.raises(ValueError):
        read_safetensors(tmp_path / "junk")


def test_registry():
    from lit_llama import registry

    assert registry.architectures() == ["Bobasun", "LLaMA", "Mugivik"]
    with pytest.raises(ValueError):
        registry.model_class("Other")
    c = registry.model_class("LLaMA").config_from_dict({"architecture": "LLaMA", "n_layer": 2, "n_head": 4, "n_embd": 64})
    assert c.n_layer == 2 and c.n_embd == 64


def test_oracle_prefix_property():
    """The logits at a position do not depend on later tokens."""
    cfg = CONFIGS["odd"]
    w = weights(cfg)
    toks = prompts(cfg, [30])[0]
    full = oracle(cfg, w, toks)
    assert np.abs(oracle(cfg, w, toks[:17]) - full[:17]).max() < 1e-9


def test_oracle_recurrence_carries_state():
    g = np.random.default_rng(0)
    q, k, v, la = g.standard_normal((9, 3)), g.standard_normal((9, 3)), g.standard_normal((9, 4)), -g.random((9, 3))
    o, s = O.gla_recurrence(q, k, v, la, np.zeros((3, 4)))
    o1, s1 = O.gla_recurrence(q[:4], k[:4], v[:4], la[:4], np.zeros((3, 4)))
    o2, s2 = O.gla_recurrence(q[4:], k[4:], v[4:], la[4:], s1)
    assert np.allclose(np.concatenate([o1, o2]), o) and np.allclose(s2, s)
