"""Small random Dovisun models on disk.  The engine harness (``Replayer``, ``make_engine``, ``write_model``,
``row_error``) is the one of ``nepevik_util``: it only speaks to the engine."""
from typing import Dict, List, Optional

import torch

from nepevik_util import Replayer, make_engine, row_error, write_model  # noqa: F401  (re-exported)


def attention(heads=4, kv_heads=2, dim=16, vdim=12, scale=0.3):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    return {"type": "attention", "mixer": {k: v for k, v in m.items() if v is not None}}


def yarn(factor=4.0, original=64, fast=6.0, slow=1.0):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def latent(heads=3, dim=8, rot_dim=4, vdim=12, kv_rank=20, q_rank=14, scale=0.35, base=40.0, scaling=None):
    rot = {"base": base, "dims": rot_dim}
    if scaling is not None:
        rot["scaling"] = scaling
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale,
         "rot": rot}
    return {"type": "latent_attention", "mixer": {k: v for k, v in m.items() if v is not None}}


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def moe(experts=5, top=2, ff=24):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def config(layers: List[dict], mlps: List[Optional[dict]], loop=None, vocab=97, width=48, eps=1e-5, embed_scale=3.7,
           softcap: Optional[float] = 6.0) -> dict:
    out = []
    for layer, mlp in zip(layers, mlps):
        entry = dict(layer)
        entry["mlp"] = mlp
        out.append(entry)
    cfg = {"architecture": "Dovisun", "embedding": {"scale": embed_scale}, "layers": out, "norm": {"eps": eps}, "vocab": vocab,
           "width": width}
    if loop is not None:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    if softcap is not None:
        cfg["logit_softcap"] = softcap
    return cfg


def random_weights(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """bf16 weights under the checkpoint's names; magnitudes chosen so that every mechanism matters: norm weights spread
    around 1, gates spread around one half, router biases that change choices, logits that reach the soft cap's bend,
    a loop projection that keeps both of its inputs."""
    g = torch.Generator().manual_seed(seed)
    width, vocab = cfg["width"], cfg["vocab"]

    def rnd(*shape, scale=1.0):
        return (torch.randn(tuple(shape), generator=g) * scale).to(torch.bfloat16)

    def lin(out, inp, gain=1.0):
        return rnd(out, inp, scale=gain / inp ** 0.5)

    sd = {"embed": rnd(vocab, width, scale=0.5), "head": lin(vocab, width, 4.0), "final.norm": rnd(width, scale=0.2) + 1.0}
    if cfg.get("loop"):
        sd["loop.in"] = torch.cat([0.8 * torch.eye(width) + 0.5 * lin(width, width).float(),
                                   0.3 * torch.eye(width) + 0.5 * lin(width, width).float()], 1).to(torch.bfloat16)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        sd[p + "norm1"] = rnd(width, scale=0.2) + 1.0
        h, d = m["heads"], m["dim"]
        dv = m.get("vdim", d)
        if layer["type"] == "latent_attention":
            dr, rank, qr = m["rot_dim"], m["kv_rank"], m["q_rank"]
            sd[p + "mix.dq"], sd[p + "mix.dq.norm"] = lin(qr, width, 2.0), rnd(qr, scale=0.3) + 1.0
            sd[p + "mix.uq"] = lin(h * (d + dr), qr, 3.0)
            sd[p + "mix.dkv"], sd[p + "mix.dkv.norm"] = lin(rank + dr, width, 2.0), rnd(rank, scale=0.3) + 1.0
            sd[p + "mix.uk"], sd[p + "mix.uv"] = lin(h * d, rank, 1.5), lin(h * dv, rank, 1.5)
            sd[p + "mix.g"] = lin(h, width, 2.0)
        else:
            kv = m.get("kv_heads", h)
            sd[p + "mix.q"], sd[p + "mix.k"], sd[p + "mix.v"] = lin(h * d, width, 2.0), lin(kv * d, width, 2.0), lin(kv * dv, width, 1.5)
        sd[p + "mix.o"] = lin(width, h * dv, 1.5)
        mlp = layer.get("mlp")
        if mlp is not None and mlp["kind"] == "dense":
            sd[p + "mlp.up"], sd[p + "mlp.down"] = lin(mlp["ff"], width), lin(width, mlp["ff"])
        elif mlp is not None:
            n, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
            for j in range(n):
                sd[p + f"mlp.e{j}.gate"], sd[p + f"mlp.e{j}.up"] = lin(ff, width, 1.5), lin(ff, width, 1.5)
                sd[p + f"mlp.e{j}.down"] = lin(width, ff, 1.5)
            sd[p + "mlp.router"], sd[p + "mlp.router.b"] = lin(n, width, 1.5), rnd(n, scale=0.8)
    return sd


# ---- whole models: where the loop lies, which layers have which feed-forward, sizes off every multiple and on them
def model_a():
    """The loop in the middle, a layer without a feed-forward, both mixers inside and outside it."""
    return config([latent(3, 8, 4, 12, 20, 14, scaling=yarn()), attention(4, 2, 16, 12), latent(2, 16, 8, 8, 24, 10, 0.25, 1000.0),
                   attention(6, 2, 10, 20, 0.4)], [dense(40), moe(5, 2, 24), None, dense(33)], loop=(1, 3, 2))


def model_b():
    """The loop over the whole model, from the first layer on; odd sizes everywhere."""
    return config([attention(3, 1, 7, 5, 0.6), latent(5, 9, 2, 3, 11, 6, 0.5, scaling=yarn(8.0, 32, 4.0, 0.5))],
                  [moe(7, 3, 9), dense(21)], loop=(0, 2, 3), vocab=53, width=22, eps=1e-6, embed_scale=0.9, softcap=2.5)


def model_c():
    """No loop, no soft cap, attention only, as many key/value heads as query heads, sizes left to their defaults."""
    return config([attention(2, None, 12, None, 0.5), attention(4, 4, 8, 30, 0.35), attention(3, 3, 24, 8)],
                  [None, moe(3, 1, 16), moe(4, 4, 8)], vocab=61, width=40, embed_scale=6.0, softcap=None)


def model_d():
    """Latent attention only, one head, the loop once and up to the last layer; routers that choose all experts."""
    return config([latent(1, 12, 2, None, 9, 5, 0.5), latent(4, 4, 6, 4, 40, 30, 0.45, 30.0, yarn(2.0, 40, 3.0, 1.0))],
                  [moe(3, 3, 20), dense(16)], loop=(1, 2, 1), vocab=70, width=32, embed_scale=2.0)


def model_e():
    """Sizes on the matrix cores' grid (multiples of 8 to 64); the loop from layer 0; routers that choose all experts."""
    return config([attention(8, 2, 64, 32, 0.125), latent(4, 32, 16, 64, 128, 48, 0.15, 10000.0, yarn(4.0, 128, 16.0, 1.0)),
                   attention(2, 1, 40, 72, 0.2)], [dense(128), moe(4, 4, 32), dense(64)], loop=(0, 2, 2), vocab=160, width=128,
                  embed_scale=11.0, softcap=20.0)


MODELS = {"a": (model_a, 21), "b": (model_b, 22), "c": (model_c, 23), "d": (model_d, 24), "e": (model_e, 25)}
