"""Small random Vufasun models on disk.  The engine harness (``Replayer``, ``make_engine``, ``write_model``,
``row_error``) is the one of ``nepevik_util``: it only speaks to the engine."""
from typing import Dict, List, Optional

import torch

from nepevik_util import Replayer, make_engine, row_error, write_model  # noqa: F401  (re-exported)


def scaling(factor=4.0, low=1.0, high=4.0, original=40):
    return {"factor": factor, "low": low, "high": high, "original": original}


def _rot(dims, base, scale=None):
    rot = {"dims": dims, "base": base}
    if scale is not None:
        rot["scaling"] = scale
    return rot


def _attn(heads, kv_heads, dim, vdim, scale, rot):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot}
    return {k: v for k, v in m.items() if v is not None}


def attention(heads=4, kv_heads=2, dim=16, vdim=12, scale=0.3, dims=10, base=60.0, rot_scaling=None):
    return {"type": "attention", "mixer": _attn(heads, kv_heads, dim, vdim, scale, _rot(dims, base, rot_scaling))}


def parallel(heads=4, kv_heads=2, dim=16, vdim=12, scale=0.3, dims=16, base=300.0, rot_scaling=None, r_heads=3, r_dim=8,
             r_vdim=12, r_dims=6, r_base=50.0, decay=(0.9, 0.98, 0.75)):
    right = {"heads": r_heads, "dim": r_dim, "rot": _rot(r_dims, r_base), "decay": list(decay)}
    if r_vdim is not None:
        right["vdim"] = r_vdim
    return {"type": "parallel", "mixer": {"left": _attn(heads, kv_heads, dim, vdim, scale, _rot(dims, base, rot_scaling)),
                                          "right": right}}


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def moe(experts=5, top=2, ff=24, shared=20):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def config(layers: List[dict], mlps: List[Optional[dict]], loop=None, streams=3, vocab=97, width=48, eps=1e-5) -> dict:
    out = []
    for layer, mlp in zip(layers, mlps):
        entry = dict(layer)
        entry["mlp"] = mlp
        out.append(entry)
    cfg = {"architecture": "Vufasun", "layers": out, "norm": {"eps": eps}, "streams": streams, "vocab": vocab, "width": width}
    if loop is not None:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


def random_weights(cfg: dict, seed: int, calm: float = 1.0) -> Dict[str, torch.Tensor]:
    """bf16 weights under the checkpoint's names; magnitudes chosen so that every mechanism matters: streams that grow apart,
    a mix that is far from symmetric, sinks of the scores' size, norm weights 0.4 around 1, router scores 0.4
    around one half.  ``calm`` < 1: smaller matrices, under which
    rounding grows less on its way through the layers."""
    g = torch.Generator().manual_seed(seed)
    width, vocab, s = cfg["width"], cfg["vocab"], cfg["streams"]

    def rnd(*shape, scale=1.0):
        return (torch.randn(tuple(shape), generator=g) * scale).to(torch.bfloat16)

    def lin(out, inp, gain=1.0):
        return rnd(out, inp, scale=calm * gain / inp ** 0.5)

    def gated(sd, name, ff, gain=1.5):
        sd[name + ".gate"], sd[name + ".up"], sd[name + ".down"] = lin(ff, width, gain), lin(ff, width, gain), lin(width, ff, gain)

    sd = {"embed": lin(vocab, width, 3.0 / calm), "final.norm": rnd(width, scale=0.3) + 1.0}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        sides = [("mix.left.", m["left"]), ("mix.right.", m["right"])] if layer["type"] == "parallel" else [("mix.", m)]
        for name, side in sides:
            h, d = side["heads"], side["dim"]
            kv, dv = (h if "right" in name else side.get("kv_heads", h)), side.get("vdim", d)
            sd[p + name + "q"], sd[p + name + "k"], sd[p + name + "v"] = lin(h * d, width, 2.0), lin(kv * d, width, 2.0), lin(kv * dv, width, 1.5)
            sd[p + name + "o"] = lin(width, h * dv, 1.5)
            if "left" in name:
                sd[p + name + "q.norm"], sd[p + name + "k.norm"] = rnd(h * d, scale=0.4) + 1.5, rnd(kv * d, scale=0.4) + 1.5
            elif "right" in name:
                sd[p + name + "g"] = lin(h * dv, width, 1.5)
            else:
                sd[p + name + "sink"] = rnd(h) + 1.5
        if layer["type"] == "parallel":
            sd[p + "mix.left.out"], sd[p + "mix.right.out"] = rnd(width, scale=0.4) + 1.0, rnd(width, scale=0.4) + 1.5
        mlp = layer.get("mlp")
        for q in ("1", "2") if mlp is not None else ("1",):
            sd[p + "norm" + q] = rnd(width, scale=0.3) + 1.0
            sd[p + f"hc{q}.in"] = rnd(s, scale=0.4) + 1.0 / s
            sd[p + f"hc{q}.out"] = rnd(s, scale=0.4) + 1.0
            sd[p + f"hc{q}.mix"] = (0.7 * torch.eye(s) + 0.3 * torch.randn(s, s, generator=g)).to(torch.bfloat16)
        if mlp is not None and mlp["kind"] == "dense":
            gated(sd, p + "mlp", mlp["ff"])
        elif mlp is not None:
            n = mlp["router"]["experts"]
            for j in range(n):
                gated(sd, p + f"mlp.e{j}", mlp["expert"]["ff"], 2.0)
            sd[p + "mlp.router"] = lin(n, width, 1.5)
            if mlp.get("shared"):
                gated(sd, p + "mlp.shared", mlp["shared"]["ff"])
    return sd


def requests(cfg: dict, seed: int) -> Dict[str, List[int]]:
    g = torch.Generator().manual_seed(seed)
    return {f"r{i}": torch.randint(0, cfg["vocab"], (n,), generator=g).tolist() for i, n in enumerate([70, 41, 18, 1, 33, 52, 150])}


# ---- whole models: where the loop lies, which layers have which feed-forward, sizes off every multiple and on them
def model_a():
    """The loop in the middle, a layer without a feed-forward, both mixers inside and outside it, scaled frequencies."""
    return config([parallel(4, 2, 16, 12, 0.3, 12, 300.0, scaling()), attention(4, 2, 16, 12),
                   parallel(3, 3, 8, 20, 0.5, 8, 100.0, None, 2, 12, 8, 12, 80.0, (0.97, 0.5)), attention(6, 2, 10, 20, 0.4, 4)],
                  [dense(40), moe(5, 2, 24, 20), None, dense(33)], loop=(1, 3, 2))


def model_b():
    """The loop over the whole model, from the first layer on; odd sizes everywhere; two streams."""
    return config([attention(3, 1, 7, 5, 0.6, 6, 20.0, scaling(8.0, 1.0, 3.0, 25)),
                   parallel(5, 1, 9, 3, 0.5, 2, 10.0, None, 3, 5, 7, 2, 9.0, (1.0, 0.9, 0.3))],
                  [moe(7, 3, 9, 11), dense(21)], loop=(0, 2, 3), streams=2, vocab=53, width=22, eps=1e-6)


def model_c():
    """No loop, one stream, as many key/value heads as query heads, sizes left to their defaults, experts without a shared one."""
    return config([attention(2, None, 12, None, 0.5, 12), parallel(4, None, 8, None, 0.35, 4, 40.0, None, 1, 16, None, 16, 90.0, (0.96,)),
                   attention(3, 3, 24, 8, 0.3, 2)], [None, moe(3, 1, 16, None), moe(4, 4, 8, 30)], streams=1, vocab=61, width=40)


def model_d():
    """Parallel layers only, one head, the loop once and up to the last layer; routers that choose all experts; five streams."""
    return config([parallel(1, 1, 12, 6, 0.5, 6, 1000.0, scaling(2.0, 1.0, 8.0, 64), 1, 6, 3, 4, 30.0, (0.85,)),
                   parallel(4, 2, 4, 40, 0.6, 4, 30.0, None, 4, 40, 36, 8, 200.0, (0.99, 0.95, 0.9, 0.6))],
                  [moe(3, 3, 20, 7), dense(16)], loop=(1, 2, 1), streams=5, vocab=70, width=32)


def model_e():
    """Sizes on the matrix cores' grid (multiples of 8 to 64); the loop from layer 0; routers that choose all experts."""
    return config([attention(8, 2, 64, 32, 0.125, 32, 5000.0),
                   parallel(4, 2, 32, 64, 0.18, 32, 10000.0, scaling(4.0, 1.0, 4.0, 128), 4, 32, 40, 16, 10000.0, (0.99, 0.97, 0.9, 0.8)),
                   attention(2, 1, 40, 72, 0.2, 24, 500.0)], [dense(128), moe(4, 4, 32, 48), dense(64)], loop=(0, 2, 2), streams=4,
                  vocab=160, width=128)


# name: (sizes, seed of weights and requests, calm); the seeds are such that no router meets two scores that rounding could swap
MODELS = {"a": (model_a, 41, 1.0), "b": (model_b, 72, 1.0), "c": (model_c, 33, 1.0), "d": (model_d, 34, 1.0), "e": (model_e, 65, 0.35)}


def load(name: str):
    """-> (configuration, weights, requests) of one of MODELS."""
    make, seed, calm = MODELS[name]
    cfg = make()
    return cfg, random_weights(cfg, seed, calm), requests(cfg, seed)
