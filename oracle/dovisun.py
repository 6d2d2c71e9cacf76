"""Plain, slow CPU statement of the Dovisun decoder -- TEST INFRASTRUCTURE ONLY.

One function per mechanism, no cache, no batching, loops over tokens and heads where they are cheap enough; nothing
here is shared with the engine's model code.  ``logits`` runs a whole token sequence and returns the logits of every
position (and, on request, the stream after every layer that is run).

Notation.  x: the stream [n, width]; U(u) = u / sqrt(mean(u^2) + eps); N(u; w) = U(u) * w.
    x_0 = scale * embedding rows
    a layer:     h = N(x; norm1);  x <- x + mixer(h) + ff(h)
    a loop:      the layers start .. stop - 1 run ``times`` times in a row; each time, before the first of them,
                 x <- W_x x + W_0 x_0     ([W_x | W_0] is one matrix)
    the output:  c tanh(head N(x; final) / c)
Weights are [out, in] and applied as W u.
"""
import math
from typing import Dict, List, Optional, Tuple

import torch


def rms_unit(u: torch.Tensor, eps: float) -> torch.Tensor:
    return u / torch.sqrt(u.pow(2).mean(-1, keepdim=True) + eps)


def rms_norm(u: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return rms_unit(u, eps) * w


def soft_cap(z: torch.Tensor, cap: Optional[float]) -> torch.Tensor:
    return cap * torch.tanh(z / cap) if cap else z


# ------------------------------------------------------------------------------------------------ rotation
def yarn_frequencies(rot: dict) -> List[float]:
    """base^(-2i / dims), slowed down by ``factor`` for the pairs that turn fewer than ``slow`` times over
    ``original`` positions, unchanged for those that turn more than ``fast`` times, a linear mix between."""
    dims, base = rot["dims"], float(rot["base"])
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if not s:
        return plain

    def pair_of(turns):                      # the (fractional) pair whose wave turns so often over ``original``
        return dims * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(pair_of(s["fast"])), 0), min(math.ceil(pair_of(s["slow"])), dims - 1)
    out = []
    for i, f in enumerate(plain):
        slowed = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * slowed + f * (1.0 - slowed))
    return out


def yarn_amplitude(rot: dict) -> float:
    s = rot.get("scaling")
    return 0.1 * math.log(s["factor"]) + 1.0 if s else 1.0


def rotate_halves(y: torch.Tensor, position: int, freqs: List[float], amplitude: float = 1.0) -> torch.Tensor:
    """y [heads, size]: pairs (i, i + len(freqs)) of the first 2 * len(freqs) coordinates turn by position * f_i and
    grow by ``amplitude``; the rest passes unchanged.  Angles are fp32 products, as the design computes them."""
    out, n = y.clone(), len(freqs)
    for i, f in enumerate(freqs):
        a = (torch.tensor(float(position), dtype=torch.float32) * torch.tensor(f, dtype=torch.float32)).to(torch.float64)
        c, s = (amplitude * torch.cos(a)).to(y.dtype), (amplitude * torch.sin(a)).to(y.dtype)
        u, v = y[:, i], y[:, i + n]
        out[:, i] = u * c - v * s
        out[:, i + n] = v * c + u * s
    return out


# ------------------------------------------------------------------------------------------------ attention
def causal_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, sink: bool = False,
                     first_position: int = 0) -> torch.Tensor:
    """q [n, H, d] at positions first_position ..; k [m, G, d], v [m, G, dv] from position 0.  -> [n, H, dv].
    Query head a reads key/value head a // (H // G).  ``sink``: the weights are exp(s_j) / (1 + sum exp(s_j))."""
    n, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(n, H, v.shape[2], dtype=q.dtype)
    for t in range(n):
        last = first_position + t
        for a in range(H):
            g = a // (H // G)
            s = (k[:last + 1, g] @ q[t, a]) * scale
            top = s.max().clamp(min=0.0) if sink else s.max()
            e = torch.exp(s - top)
            p = e / (e.sum() + (torch.exp(-top) if sink else 0.0))
            out[t, a] = p @ v[:last + 1, g]
    return out


def attention_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    """Grouped query heads, no positions in the scores, unit queries and keys, a sink in the softmax."""
    n, H, d = h.shape[0], m["heads"], m["dim"]
    G, dv = m.get("kv_heads", H), m.get("vdim", d)
    q = rms_unit((h @ w["q"].T).view(n, H, d), eps)
    k = rms_unit((h @ w["k"].T).view(n, G, d), eps)
    v = (h @ w["v"].T).view(n, G, dv)
    out = causal_attention(q, k, v, m["scale"], sink=True)
    return out.reshape(n, H * dv) @ w["o"].T


def latent_attention_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    """Queries through a latent of their own; keys and values of all heads from another latent, plus one rotated key
    part that the heads share; one sigmoid gate per head."""
    n, H, d, dr, rank = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    dv = m.get("vdim", d)
    freqs, amp = yarn_frequencies(m["rot"]), yarn_amplitude(m["rot"])
    c_q = rms_norm(h @ w["dq"].T, w["dq.norm"], eps)
    q = (c_q @ w["uq"].T).view(n, H, d + dr)
    down = h @ w["dkv"].T
    c = rms_norm(down[:, :rank], w["dkv.norm"], eps)
    k_rot = torch.stack([rotate_halves(down[t:t + 1, rank:], t, freqs, amp)[0] for t in range(n)])
    q_rot = torch.stack([rotate_halves(q[t, :, d:], t, freqs, amp) for t in range(n)])
    k_plain = (c @ w["uk"].T).view(n, H, d)
    v = (c @ w["uv"].T).view(n, H, dv)
    keys = torch.cat([k_plain, k_rot.unsqueeze(1).expand(n, H, dr)], -1)
    queries = torch.cat([q[:, :, :d], q_rot], -1)
    out = causal_attention(queries, keys, v, m["scale"])
    gate = torch.sigmoid(h @ w["g"].T)
    return (out * gate.unsqueeze(-1)).reshape(n, H * dv) @ w["o"].T


# ------------------------------------------------------------------------------------------------ feed-forward
def dense_ff(h: torch.Tensor, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    return torch.relu(h @ w["up"].T).pow(2) @ w["down"].T


def route(h: torch.Tensor, router: torch.Tensor, bias: torch.Tensor, top: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """-> (chosen [n, top], weights [n, top]): the largest logits; their softmax among themselves."""
    z = h @ router.T + bias
    best, chosen = torch.topk(z, top, dim=-1)
    return chosen, torch.softmax(best, -1)


def expert(h: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor) -> torch.Tensor:
    z = h @ gate.T
    return (z * torch.sigmoid(z) * (h @ up.T)) @ down.T


def moe_ff(h: torch.Tensor, w: Dict[str, torch.Tensor], mlp: dict) -> torch.Tensor:
    chosen, weights = route(h, w["router"], w["router.b"], mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, p in zip(chosen[t].tolist(), weights[t]):
            out[t] += p * expert(h[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"])
    return out


def feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor], mlp: Optional[dict]) -> torch.Tensor:
    if mlp is None:
        return torch.zeros_like(h)
    if mlp["kind"] == "dense":
        return dense_ff(h, w)
    if mlp["kind"] == "moe":
        return moe_ff(h, w, mlp)
    raise ValueError(mlp["kind"])


# ------------------------------------------------------------------------------------------------ the whole model
def layer_runs(cfg: dict) -> List[Tuple[int, bool]]:
    """-> [(layer, first of a pass of the loop?)] in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    body = [(i, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return [(i, False) for i in range(loop["start"])] + body * loop["times"] + [(i, False) for i in range(loop["stop"], n)]


def logits(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64,
           keep_streams: bool = False):
    """-> logits [n, vocab] (and the stream after every layer that was run)."""
    W = {k: (v.to(dtype) if v.dtype.is_floating_point else v) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]

    def sub(prefix):
        return {k[len(prefix):]: v for k, v in W.items() if k.startswith(prefix)}

    x0 = W["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
    x, streams = x0, []
    for i, first in layer_runs(cfg):
        if first:
            x = torch.cat([x, x0], -1) @ W["loop.in"].T
        layer, p = cfg["layers"][i], f"l{i}."
        h = rms_norm(x, W[p + "norm1"], eps)
        if layer["type"] == "attention":
            a = attention_mixer(h, sub(p + "mix."), layer["mixer"], eps)
        elif layer["type"] == "latent_attention":
            a = latent_attention_mixer(h, sub(p + "mix."), layer["mixer"], eps)
        else:
            raise ValueError(layer["type"])
        x = x + (a + feed_forward(h, sub(p + "mlp."), layer.get("mlp")))
        streams.append(x)
    out = soft_cap(rms_norm(x, W["final.norm"], eps) @ W["head"].T, cfg.get("logit_softcap"))
    return (out, streams) if keep_streams else out
