"""Plain, slow CPU statement of the Vufasun decoder -- TEST INFRASTRUCTURE ONLY.

One function per mechanism, no cache, no batching, loops over tokens and heads where they are cheap enough; nothing
here is shared with the engine's model code.  ``logits`` runs a whole token sequence and returns the logits of every
position (and, on request, the sum of the streams after every layer that is run).

Notation.  X: the streams [s, n, width]; U(u) = u / sqrt(mean(u^2) + eps); N(u; w) = U(u) * w.
    X_a = embedding rows, the same in all s streams
    a sublayer f with its a (reads), M (stream to stream, [from, to]) and b (writes):
        y = f(N(sum_i a_i X_i)),   X_j <- sum_i M_ij X_i + b_j y      (all j at once)
    a layer: the mixer, then the feed-forward (if it has one);  a loop runs some neighbouring layers several times
    the logits: E N(sum_i X_i; final), E the embedding table
Weights are [out, in] and applied as W u.
"""
import math
from typing import Dict, List, Optional, Tuple

import torch


def rms_unit(u: torch.Tensor, eps: float) -> torch.Tensor:
    return u / torch.sqrt(u.pow(2).mean(-1, keepdim=True) + eps)


def rms_norm(u: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return rms_unit(u, eps) * w


# ------------------------------------------------------------------------------------------------ streams
def read_streams(X: torch.Tensor, reads: torch.Tensor) -> torch.Tensor:
    """X [s, n, width], reads [s] -> [n, width]."""
    return sum(reads[i] * X[i] for i in range(X.shape[0]))


def write_streams(X: torch.Tensor, mix: torch.Tensor, writes: torch.Tensor, y: torch.Tensor) -> torch.Tensor:
    """mix [from, to], writes [s], y [n, width] -> the new streams, every one made from the old ones."""
    s = X.shape[0]
    return torch.stack([sum(mix[i, j] * X[i] for i in range(s)) + writes[j] * y for j in range(s)])


# ------------------------------------------------------------------------------------------------ rotation
def rotary_frequencies(rot: dict) -> List[float]:
    """base^(-2i / dims); with ``scaling`` waves longer than original / low are slowed by factor, those shorter than
    original / high are kept, and between the two the frequency is a mix, linear in original / wavelength."""
    out = []
    s = rot.get("scaling")
    for i in range(rot["dims"] // 2):
        f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
        if s:
            turns = s["original"] * f / (2.0 * math.pi)          # original / wavelength
            kept = min(1.0, max(0.0, (turns - s["low"]) / (s["high"] - s["low"])))
            f = kept * f + (1.0 - kept) * f / s["factor"]
        out.append(f)
    return out


def rotate_halves(y: torch.Tensor, position: int, freqs: List[float]) -> torch.Tensor:
    """y [heads, size]: pairs (i, i + len(freqs)) of the first 2 * len(freqs) coordinates turn by position * f_i; the rest
    passes unchanged.  Angles are fp32 products, as the design computes them."""
    out, n = y.clone(), len(freqs)
    for i, f in enumerate(freqs):
        a = (torch.tensor(float(position), dtype=torch.float32) * torch.tensor(f, dtype=torch.float32)).to(torch.float64)
        c, s = torch.cos(a).to(y.dtype), torch.sin(a).to(y.dtype)
        u, v = y[:, i], y[:, i + n]
        out[:, i] = u * c - v * s
        out[:, i + n] = v * c + u * s
    return out


def rotate_all(y: torch.Tensor, freqs: List[float]) -> torch.Tensor:
    """y [n, heads, size] at positions 0 .. n - 1."""
    return torch.stack([rotate_halves(y[t], t, freqs) for t in range(y.shape[0])])


# ------------------------------------------------------------------------------------------------ attention
def causal_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, sink: Optional[torch.Tensor] = None,
                     first_position: int = 0) -> torch.Tensor:
    """q [n, H, d] at positions first_position ..; k [m, G, d], v [m, G, dv] from position 0.  -> [n, H, dv].
    Query head a reads key/value head a // (H // G).  ``sink`` [H]: the weights are exp(s_j) / (exp(sink_a) + sum exp(s_j))."""
    n, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(n, H, v.shape[2], dtype=q.dtype)
    for t in range(n):
        last = first_position + t
        for a in range(H):
            g = a // (H // G)
            s = (k[:last + 1, g] @ q[t, a]) * scale
            top = s.max() if sink is None else torch.maximum(s.max(), sink[a])
            e = torch.exp(s - top)
            p = e / (e.sum() + (torch.exp(sink[a] - top) if sink is not None else 0.0))
            out[t, a] = p @ v[:last + 1, g]
    return out


def _head_sizes(m: dict) -> Tuple[int, int, int, int]:
    H, d = m["heads"], m["dim"]
    return H, m.get("kv_heads", H), d, m.get("vdim", d)


def attention_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict) -> torch.Tensor:
    """Grouped query heads, rotated queries and keys, a learned sink per head."""
    n = h.shape[0]
    H, G, d, dv = _head_sizes(m)
    f = rotary_frequencies(m["rot"])
    q = rotate_all((h @ w["q"].T).view(n, H, d), f)
    k = rotate_all((h @ w["k"].T).view(n, G, d), f)
    v = (h @ w["v"].T).view(n, G, dv)
    return causal_attention(q, k, v, m["scale"], w["sink"]).reshape(n, H * dv) @ w["o"].T


def normed_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    """Grouped query heads; one RMS norm over ALL rows of q (and of k), then the rotation; plain softmax."""
    n = h.shape[0]
    H, G, d, dv = _head_sizes(m)
    f = rotary_frequencies(m["rot"])
    q = rotate_all(rms_norm(h @ w["q"].T, w["q.norm"], eps).view(n, H, d), f)
    k = rotate_all(rms_norm(h @ w["k"].T, w["k.norm"], eps).view(n, G, d), f)
    v = (h @ w["v"].T).view(n, G, dv)
    return causal_attention(q, k, v, m["scale"]).reshape(n, H * dv) @ w["o"].T


# ------------------------------------------------------------------------------------------------ retention
def retention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: List[float],
              state: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """q, k [n, H, d], v [n, H, dv]: S <- decay_a S + k v^T, o = S^T q, token by token.  -> (o [n, H, dv], S [H, d, dv])."""
    n, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    lam = torch.tensor(decay, dtype=q.dtype).view(H, 1, 1)
    out = torch.zeros(n, H, v.shape[2], dtype=q.dtype)
    for t in range(n):
        S = lam * S + k[t].unsqueeze(2) * v[t].unsqueeze(1)
        out[t] = (S * q[t].unsqueeze(2)).sum(1)
    return out, S


def retention_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    n = h.shape[0]
    H, d = m["heads"], m["dim"]
    dv = m.get("vdim", d)
    f = rotary_frequencies(m["rot"])
    q = rotate_all((h @ w["q"].T).view(n, H, d), f)
    k = rotate_all((h @ w["k"].T).view(n, H, d), f) * d ** -0.5
    v = (h @ w["v"].T).view(n, H, dv)
    o, _ = retention(q, k, v, m["decay"])
    z = h @ w["g"].T
    return (rms_unit(o, eps).reshape(n, H * dv) * (z * torch.sigmoid(z))) @ w["o"].T


def parallel_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float) -> torch.Tensor:
    """Both mixers on the same input; the mean of their normed outputs."""
    side = {s: {k[len(s) + 1:]: v for k, v in w.items() if k.startswith(s + ".")} for s in ("left", "right")}
    left = normed_attention(h, side["left"], m["left"], eps)
    right = retention_mixer(h, side["right"], m["right"], eps)
    return 0.5 * (rms_norm(left, w["left.out"], eps) + rms_norm(right, w["right.out"], eps))


# ------------------------------------------------------------------------------------------------ feed-forward
def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def gated_ff(h: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor, act) -> torch.Tensor:
    return (act(h @ gate.T) * (h @ up.T)) @ down.T


def route(h: torch.Tensor, router: torch.Tensor, top: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """-> (chosen [n, top], weights [n, top]): the largest sigmoid scores, as they are."""
    best, chosen = torch.topk(torch.sigmoid(h @ router.T), top, dim=-1)
    return chosen, best


def moe_ff(h: torch.Tensor, w: Dict[str, torch.Tensor], mlp: dict) -> torch.Tensor:
    """An expert's weight multiplies what the expert READS."""
    chosen, weights = route(h, w["router"], mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, p in zip(chosen[t].tolist(), weights[t]):
            out[t] += gated_ff(p * h[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], silu)
    if mlp.get("shared"):
        out = out + gated_ff(h, w["shared.gate"], w["shared.up"], w["shared.down"], silu)
    return out


def feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor], mlp: dict) -> torch.Tensor:
    if mlp["kind"] == "dense":
        return gated_ff(h, w["gate"], w["up"], w["down"], gelu_tanh)
    if mlp["kind"] == "moe":
        return moe_ff(h, w, mlp)
    raise ValueError(mlp["kind"])


# ------------------------------------------------------------------------------------------------ the whole model
def layer_order(cfg: dict) -> List[int]:
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    body = list(range(loop["start"], loop["stop"]))
    return list(range(loop["start"])) + body * loop["times"] + list(range(loop["stop"], n))


def logits(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64,
           keep_streams: bool = False):
    """-> logits [n, vocab] (and the sum of the streams after every layer that was run)."""
    W = {k: (v.to(dtype) if v.dtype.is_floating_point else v) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]

    def sub(prefix):
        return {k[len(prefix):]: v for k, v in W.items() if k.startswith(prefix)}

    x0 = W["embed"][torch.tensor(tokens)]
    X, kept = torch.stack([x0] * cfg["streams"]), []
    for i in layer_order(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        h = rms_norm(read_streams(X, W[p + "hc1.in"]), W[p + "norm1"], eps)
        if layer["type"] == "attention":
            y = attention_mixer(h, sub(p + "mix."), layer["mixer"])
        elif layer["type"] == "parallel":
            y = parallel_mixer(h, sub(p + "mix."), layer["mixer"], eps)
        else:
            raise ValueError(layer["type"])
        X = write_streams(X, W[p + "hc1.mix"], W[p + "hc1.out"], y)
        if layer.get("mlp") is not None:
            h = rms_norm(read_streams(X, W[p + "hc2.in"]), W[p + "norm2"], eps)
            X = write_streams(X, W[p + "hc2.mix"], W[p + "hc2.out"], feed_forward(h, sub(p + "mlp."), layer["mlp"]))
        kept.append(X.sum(0))
    out = rms_norm(X.sum(0), W["final.norm"], eps) @ W["embed"].T
    return (out, kept) if keep_streams else out
