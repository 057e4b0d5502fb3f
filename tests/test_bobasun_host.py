"""Bobasun without a GPU: configuration reading, tensor checks, growing K / V rows, work tables, and the oracle's own
consistency."""
import copy
import json

import numpy as np
import pytest
import torch

from oracle import bobasun_np as O
from tests.bobasun_cases import CONFIGS, build, errors, oracle, prompts, weights


def _cfg(d):
    from lit_llama.bobasun import BobasunConfig

    return BobasunConfig.from_dict(d)


@pytest.mark.parametrize("name", list(CONFIGS))
def test_config_and_tensors(name):
    cfg = CONFIGS[name]
    c = _cfg(json.loads(json.dumps(cfg)))
    assert c.n_layer == len(cfg["layers"]) and c.vocab_size == cfg["vocab"] and c.streams == cfg["streams"]
    w = weights(cfg)
    build(cfg, w, torch.float32, "cpu")
    bad = dict(w)
    bad.pop("l0.mix.vmix" if "l0.mix.vmix" in w else "l0.hc1.mix")
    with pytest.raises(ValueError):
        build(cfg, bad, torch.float32, "cpu")
    with pytest.raises(ValueError, match="unexpected"):
        build(cfg, dict(w, extra=w["embed"]), torch.float32, "cpu")
    with pytest.raises(ValueError, match="shape"):
        build(cfg, dict(w, **{"final.norm": w["final.norm"][1:]}), torch.float32, "cpu")


def test_config_errors():
    def broken(edit):
        d = copy.deepcopy(CONFIGS["odd"])
        edit(d)
        with pytest.raises(ValueError):
            _cfg(d)

    broken(lambda d: d.update(extra=1))
    broken(lambda d: d.pop("streams"))
    broken(lambda d: d["layers"][0].update(type="other"))
    broken(lambda d: d["layers"][0]["mixer"]["rot"].update(dims=5))
    broken(lambda d: d["layers"][0]["mixer"]["rot"].update(dims=12))  # more than a head has
    broken(lambda d: d["layers"][0]["mixer"].update(kv_heads=2))  # 3 query heads
    broken(lambda d: d["layers"][3]["mixer"].update(vdim=8))  # mixes values of another size
    broken(lambda d: d["layers"][0]["mlp"].update(kind="other"))
    broken(lambda d: d["layers"][0]["mlp"].pop("limit"))


def test_optional_keys():
    d = copy.deepcopy(CONFIGS["odd"])
    d["layers"][0]["mixer"].pop("v_mix")
    d["layers"][0]["mixer"]["rot"].pop("scaling")
    d["layers"][1].pop("mlp")
    c = _cfg(d)
    assert c.layers[0].mixer.rot_factor == 1.0 and not c.layers[0].mixer.v_mix and c.layers[1].ff is None


def test_first_mixing_layer():
    from lit_llama.bobasun import Bobasun

    m = Bobasun(_cfg(CONFIGS["odd"]))
    assert [mx.first is m.mixers[1] for mx in m.mixers] == [False, True, False, True, True]
    m = build(CONFIGS["odd"], weights(CONFIGS["odd"]), torch.float32, "cpu")
    assert [mx.lam is not None for mx in m.mixers] == [False, False, False, True, True]


def test_rows_grow_and_slots():
    m = build(CONFIGS["odd"], weights(CONFIGS["odd"]), torch.float32, "cpu")
    st = m.new_state(2)
    assert set(st.ring_rows.values()) == {0}
    a = st.alloc(2)
    assert st.ensure(5) and not st.ensure(200) and st.ring_rows[0] == 256
    st.ring[3][a[1], 17] = 2.5
    assert st.ensure(257) and st.ring_rows[0] == 512 and st.ring[3].shape[1] == 512
    assert float(st.ring[3][a[1], 17].min()) == 2.5 and float(st.ring[3][a[0]].abs().max()) == 0.0
    st.release(a)
    st.reserve(7)
    assert st.ring[0].shape[:2] == (7, 512)
    fixed = m.new_state(1, 40)
    assert fixed.ring_rows[0] == 40 and not fixed.ensure(40)
    with pytest.raises(ValueError):
        fixed.ensure(41)


def test_pairs_cover_every_row_once():
    from lit_llama.state import Rows

    lens, starts = [1, 130, 64, 300], [5, 0, 700, 0]
    r = Rows.packed([[0] * n for n in lens], starts, [3, 0, 1, 2], "cpu")
    n, tab = r.pairs(64)
    seen, tab = np.zeros(sum(lens), int), tab.view(-1, 2, 3).tolist()
    assert n == len(tab)
    row0 = np.concatenate([[0], np.cumsum(lens)])
    for late, early in tab:
        assert late[1] > 0
        for r0, k, b in (late, early):
            assert 0 <= k <= 64 and (k == 0 or row0[b] <= r0 and r0 + k <= row0[b + 1])
            seen[r0:r0 + k] += 1
    assert (seen == 1).all()


def test_interleaved_unit_weights():
    from lit_llama.mixers import PackedLinear

    g, u = torch.randn(5, 3), torch.randn(5, 3)
    lin = PackedLinear([g, u], torch.float32, "cpu", [torch.arange(5.0), None], unit=(1.0, 1.7))
    assert lin.Np == 16 and lin.out_columns == 8
    assert torch.equal(lin.w[0:10:2, :3], g) and torch.equal(lin.w[1:10:2, :3], u) and float(lin.w[10:].abs().max()) == 0.0
    assert lin.bias.tolist() == [0, 0, 1, 0, 2, 0, 3, 0, 4, 0] + [0] * 6


def test_oracle_prefix_property():
    cfg = CONFIGS["odd"]
    w = weights(cfg)
    toks = prompts(cfg, [30])[0]
    full = oracle(cfg, w, toks)
    assert np.abs(oracle(cfg, w, toks[:17]) - full[:17]).max() < 1e-9


def test_oracle_mechanisms_matter():
    """Each mechanism left out changes the logits far beyond the tolerance of the float32 device tests."""
    cfg = CONFIGS["tiled"]
    w = weights(cfg)
    toks = prompts(cfg, [40])[0]
    ref = oracle(cfg, w, toks)

    def edited(edit):
        c = copy.deepcopy(cfg)
        edit(c)
        return errors(oracle(c, w, toks), ref)[0]

    assert edited(lambda c: c["layers"][3]["mixer"].update(v_mix=False)) > 1e-3
    assert edited(lambda c: c["layers"][0]["mixer"].update(v_mix=False)) > 1e-3  # another layer's values are the first
    assert edited(lambda c: c["layers"][1]["mlp"].update(limit=1.0)) > 1e-3
    assert edited(lambda c: c["embedding"].update(scale=1.0)) > 1e-3
    for name in ("l0.hc1.mix", "l3.hc2.mix"):
        t = dict(w, **{name: w[name].T})
        assert errors(oracle(cfg, t, toks), ref)[0] > 1e-3
    for name in ("l0.mix.v.b", "l1.mix.o.b", "l0.mlp.gate.b", "l3.mlp.down.b", "l1.mix.g"):
        t = dict(w, **{name: 0 * w[name]})
        assert errors(oracle(cfg, t, toks), ref)[0] > 1e-3, name


def test_oracle_sink():
    q, k, v = np.zeros((3, 2)), np.ones((3, 2)), np.ones((3, 4))
    assert np.allclose(O.sink_attention(q, k, v, 1.0)[:, 0], [1 / 2, 2 / 3, 3 / 4])  # scores 0: one more in the denominator
