"""Small Bobasun configurations and weights for the tests (no checkpoint, no golden file)."""
import numpy as np
import torch

from oracle import bobasun_np as O
from tests.mugivik_cases import TOL, check, errors, prompts  # noqa: F401  (shared with the tests of this model)


def layer(heads, kv_heads, dim, vdim, ff, rot_dims=None, scale=None, base=900.0, factor=1.0, v_mix=False, limit=2.0):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5, "v_mix": v_mix,
         "rot": {"base": base, "dims": rot_dims or dim, "scaling": {"factor": factor}}}
    return {"type": "attention", "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}


def config(width, vocab, streams, layers, scale=3.0, eps=1e-5):
    return {"architecture": "Bobasun", "width": width, "vocab": vocab, "streams": streams, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "layers": layers}


CONFIGS = {
    # sizes that fit no tile, every layer different, values mixed in layers 1, 3 and 4
    "odd": config(75, 101, 3, [layer(3, 1, 10, 14, 40, 6, base=50.0, factor=2.5), layer(6, 2, 7, 9, None, 4, v_mix=True),
                               layer(2, 2, 5, 3, 24, 2, limit=0.5), layer(4, 2, 12, 9, 56, v_mix=True, factor=0.5),
                               layer(2, 2, 8, 9, 30, v_mix=True)]),
    "ones": config(24, 33, 1, [layer(1, 1, 2, 1, 1, v_mix=True), layer(1, 1, 2, 1, 8, v_mix=True)], scale=1.0),
    # sizes the tiled kernels take
    "tiled": config(192, 300, 2, [layer(6, 2, 48, 24, 320, 32, v_mix=True, factor=8.0), layer(6, 2, 48, 24, 136, 16, v_mix=True),
                                  layer(4, 4, 32, 40, None), layer(8, 2, 40, 24, 264, v_mix=True, base=1e6)], scale=0.5),
    "wide": config(1024, 384, 4, [layer(20, 1, 128, 96, 512, v_mix=True), layer(20, 1, 96, 96, 1024, 64, v_mix=True),
                                  layer(4, 1, 136, 168, 384)], eps=1e-6),
    "many": config(136, 90, 6, [layer(4, 2, 64, 64, 160, v_mix=True), layer(4, 2, 64, 64, 160, v_mix=True)]),
}


def weights(cfg, seed=0):
    """Tensors by name, bf16-representable float32."""
    from lit_llama.bobasun import Bobasun, BobasunConfig

    g, S = np.random.default_rng(seed), cfg["streams"]
    out = {}
    for name, shape in Bobasun(BobasunConfig.from_dict(cfg)).tensor_shapes().items():
        if ".hc" in name:
            a = 0.3 * g.standard_normal(shape) + (0.8 * np.eye(S) if name.endswith("mix") else 1.0 / S if name.endswith("in") else 0.7)
        elif name.endswith(".vmix"):
            a = np.asarray(g.uniform(0.2, 0.8))
        elif len(shape) == 1:
            a = 0.2 * g.standard_normal(shape) + (0.0 if name.endswith(".b") else 1.0)
        else:
            a = g.standard_normal(shape) * shape[1] ** -0.5
        out[name] = torch.tensor(a, dtype=torch.float32).to(torch.bfloat16).float().numpy()
    return out


def build(cfg, w, dtype, device="cuda"):
    from lit_llama.bobasun import Bobasun, BobasunConfig

    return Bobasun.from_tensors(BobasunConfig.from_dict(cfg), {k: torch.from_numpy(np.array(v)) for k, v in w.items()}, dtype,
                                device)


def oracle(cfg, w, tokens):
    return O.forward(tokens, cfg, w)
