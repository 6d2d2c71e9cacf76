"""Vufasun: a decoder whose layers are listed one by one in its config.json, whose residual is several parallel streams,
and a block of whose layers may run several times in a row with the same weights.

Each entry of ``layers`` names the layer's token mixer -- ``attention`` (grouped query heads, rotary embedding, a learned
sink per head in the softmax) or ``parallel`` (two mixers on the same input: ``left``, attention whose queries and keys get
one RMS norm over all heads before the rotation, and ``right``, retention: linear attention with one constant decay per
head) -- with the mixer's sizes, and its feed-forward: ``dense`` (down(gelu_tanh(gate h) * up h)), ``moe`` (sigmoid router;
an expert's score multiplies what the expert reads; experts and the shared expert down(silu(gate h) * up h)) or none.

With N(u; w) = u / rms(u) * w, the streams x_1 .. x_s (all the embedding row at the start), and per sublayer f its numbers
a (reads), M (stream to stream, [from, to]), b (writes):
    y = f(N(sum_i a_i x_i));  x_j <- sum_i M_ij x_i + b_j y     (all j from the old streams)
    a layer:          the mixer, then the feed-forward;  ``loop``: layers start .. stop - 1 run ``times`` times in a row
    a parallel mixer: (N(left; w_l) + N(right; w_r)) / 2
    the logits:       E N(sum_i x_i), E the embedding table
The streams are fp32.  Between two sublayers there is one kernel (``HyperConnection.step``): the output's write to all
streams, their mix, the next sublayer's read and its norm (behind a parallel mixer also the two output norms and their
mean).  All projections that a mixer's input takes are one GEMM.
Steps arrive in the ragged layout (``InputMetadata.ragged``): any mix of prompt portions and decoded tokens.

The worker allocates what ``cache_layout`` asks for per layer RUN: a layer that runs several times has pages, and a state
slot per sequence, of its own for every pass.
"""
from typing import Dict, List, Optional, Tuple

import torch
import torch.nn as nn

from ..input_metadata import InputMetadata
from ..layers.attention import RotaryPagedAttention
from ..layers.basic import GatedActivation, HyperConnection, OffsetRMSNorm, scaled_rotary_frequencies
from ..layers.linear import LinearMethodBase, MergedColumnParallelLinear, RowParallelLinear
from ..layers.moe import GroupRoutedExperts
from ..layers.recurrent import RetentionMixer
from ..layers.sampler import Sampler, SamplingMetadata
from ..layers.vocab_parallel_embedding import VocabParallelEmbedding
from ..parallel_state import get_tensor_model_parallel_world_size
from .layer_list import layer_runs

_MIXERS = ("attention", "parallel")


def _attention_of(layer: dict) -> dict:
    """The softmax attention's part of a layer's mixer."""
    return layer["mixer"]["left"] if layer["type"] == "parallel" else layer["mixer"]


def _sizes(m: dict) -> Tuple[int, int, int, int]:
    """Query heads, key/value heads, key size, value size."""
    return m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m.get("vdim", m["dim"])


def _frequencies(m: dict) -> torch.Tensor:
    rot = m.get("rot")
    return scaled_rotary_frequencies(rot["dims"], rot["base"], rot.get("scaling")) if rot else torch.zeros(0)


def normalize_config(raw: dict) -> dict:
    """The engine's generic geometry keys for a Vufasun config.json."""
    cfg = dict(raw)
    cfg["architecture"] = "vufasun"
    cfg["vocab_size"] = raw["vocab"]
    cfg["hidden_size"] = raw["width"]
    cfg["num_hidden_layers"] = len(layer_runs(raw))
    first = _sizes(_attention_of(raw["layers"][0])) if raw["layers"] else (1, 1)
    cfg["num_attention_heads"], cfg["num_key_value_heads"] = first[:2]
    cfg.setdefault("max_position_embeddings", 1 << 20)       # angles come from fp32 positions: no table to outgrow
    cfg.setdefault("torch_dtype", "bfloat16")
    return cfg


class _InputProjection(MergedColumnParallelLinear):
    """One GEMM for all projections of a mixer's input; ``parts`` of its result are column ranges.  The columns are padded
    to whole 32-byte runs so that every row begins on one."""

    def __init__(self, width: int, sizes: List[int], dtype, linear_method) -> None:
        pad = -sum(sizes) % 16
        super().__init__(width, sizes + ([pad] if pad else []), False, dtype, linear_method)
        self.part_sizes = sizes

    def parts(self, h: torch.Tensor) -> List[torch.Tensor]:
        proj, cols, lo = self(h), [], 0
        for n in self.part_sizes:
            cols.append(proj[:, lo:lo + n])
            lo += n
        return cols

    def load_parts(self, matrices: List[torch.Tensor]) -> None:
        self.weight.data.zero_()                               # the padding's rows
        self.weight.data[:sum(self.part_sizes)].copy_(torch.cat(matrices, 0))


class AttentionMixer(nn.Module):
    def __init__(self, width: int, m: dict, eps: float, dtype, linear_method) -> None:
        super().__init__()
        h, g, d, dv = _sizes(m)
        self.in_proj = _InputProjection(width, [h * d, g * d, g * dv], dtype, linear_method)
        self.attn = RotaryPagedAttention(h, g, d, dv, m["scale"], _frequencies(m), sink=True)
        self.o_proj = RowParallelLinear(h * dv, width, False, dtype, linear_method)

    def forward(self, h: torch.Tensor, positions: torch.Tensor, cache: List[torch.Tensor], md: InputMetadata) -> dict:
        """-> the output as ``HyperConnection.step`` takes it."""
        q, k, v = self.in_proj.parts(h)
        return {"a": self.o_proj(self.attn(q, k, v, positions, cache[0], cache[1], md))}

    def load_named(self, w: Dict[str, torch.Tensor]) -> None:
        self.in_proj.load_parts([w["q"], w["k"], w["v"]])
        self.attn.sink.data.copy_(w["sink"].float())
        self.o_proj.weight.data.copy_(w["o"])

    @torch.no_grad()
    def random_init(self, rnd) -> None:
        rnd(self.attn.sink, 1.0)


class ParallelMixer(nn.Module):
    """Attention (``left``) and retention (``right``) on the same input: one input GEMM (left q | k | v, right q | k | v |
    gate), one kernel that prepares the rotated operands of both, an output projection per side; the norms of the two
    outputs and their mean are part of the write to the streams."""

    def __init__(self, width: int, m: dict, eps: float, dtype, linear_method) -> None:
        super().__init__()
        left, right = m["left"], m["right"]
        h, g, d, dv = _sizes(left)
        rh, _, rd, rdv = _sizes(right)
        self.in_proj = _InputProjection(width, [h * d, g * d, g * dv, rh * rd, rh * rd, rh * rdv, rh * rdv], dtype, linear_method)
        self.attn = RotaryPagedAttention(h, g, d, dv, left["scale"], _frequencies(left), whole_norm_eps=eps)
        self.retention = RetentionMixer(rh, rd, rdv, right["decay"], _frequencies(right), eps)
        self.left_o = RowParallelLinear(h * dv, width, False, dtype, linear_method)
        self.right_o = RowParallelLinear(rh * rdv, width, False, dtype, linear_method)
        self.left_norm = nn.Parameter(torch.ones(width, dtype=torch.float32), requires_grad=False)
        self.right_norm = nn.Parameter(torch.ones(width, dtype=torch.float32), requires_grad=False)

    def forward(self, h: torch.Tensor, positions: torch.Tensor, cache: List[torch.Tensor], md: InputMetadata) -> dict:
        q, k, v, rq, rk, rv, gate = self.in_proj.parts(h)
        linear = self.retention.operands(rq, rk)
        q32 = self.attn.prepare(q, k, v, positions, cache[0], cache[1], md, linear)
        left = self.left_o(self.attn.attend(q32, cache[0], cache[1], md, h.dtype))
        right = self.right_o(self.retention.core(linear[0], linear[1], rv, gate, cache[2], md))
        return {"a": left, "b": right, "norms": (self.left_norm.data, self.right_norm.data), "blend": 0.5}

    def load_named(self, w: Dict[str, torch.Tensor]) -> None:
        self.in_proj.load_parts([w["left.q"], w["left.k"], w["left.v"], w["right.q"], w["right.k"], w["right.v"], w["right.g"]])
        self.attn.q_norm.data.copy_(w["left.q.norm"].float())
        self.attn.k_norm.data.copy_(w["left.k.norm"].float())
        self.left_o.weight.data.copy_(w["left.o"])
        self.right_o.weight.data.copy_(w["right.o"])
        self.left_norm.data.copy_(w["left.out"].float())
        self.right_norm.data.copy_(w["right.out"].float())

    @torch.no_grad()
    def random_init(self, rnd) -> None:
        for t in (self.attn.q_norm, self.attn.k_norm, self.left_norm, self.right_norm):
            rnd(t, 0.1, 1.0)


class DenseFeedForward(nn.Module):
    def __init__(self, width: int, ff: int, dtype, linear_method) -> None:
        super().__init__()
        self.gate_up = MergedColumnParallelLinear(width, [ff, ff], False, dtype, linear_method)
        self.act = GatedActivation("gelu_tanh")
        self.down = RowParallelLinear(ff, width, False, dtype, linear_method)

    def forward(self, h: torch.Tensor) -> dict:
        return {"a": self.down(self.act(self.gate_up(h)))}

    def load_named(self, w: Dict[str, torch.Tensor]) -> None:
        self.gate_up.weight.data.copy_(torch.cat([w["gate"], w["up"]], 0))
        self.down.weight.data.copy_(w["down"])


class ExpertFeedForward(nn.Module):
    def __init__(self, width: int, mlp: dict, dtype, linear_method) -> None:
        super().__init__()
        r = mlp["router"]
        self.experts = GroupRoutedExperts(width, r["experts"], r["top"], mlp["expert"]["ff"], (mlp.get("shared") or {}).get("ff"),
                                          1, 1, 1.0, dtype, linear_method, score="sigmoid", normalize=False,
                                          activation="clamped_glu", glu_alpha=1.0, glu_shift=0.0, router_dtype=dtype,
                                          weigh_input=True)

    def forward(self, h: torch.Tensor) -> dict:
        shared, routed = self.experts(h)
        return {"a": shared, "c": routed}

    def load_named(self, w: Dict[str, torch.Tensor]) -> None:
        self.experts.load_named(w)


def _feed_forward(width: int, mlp: dict, index: int, dtype, linear_method):
    if mlp["kind"] == "dense":
        return DenseFeedForward(width, int(mlp["ff"]), dtype, linear_method)
    if mlp["kind"] == "moe":
        return ExpertFeedForward(width, mlp, dtype, linear_method)
    raise ValueError(f"layer {index}: unknown feed-forward kind {mlp['kind']!r}")


class VufasunLayer(nn.Module):
    def __init__(self, cfg: dict, index: int, dtype, linear_method) -> None:
        super().__init__()
        layer, width, eps, streams = cfg["layers"][index], cfg["width"], cfg["norm"]["eps"], cfg.get("streams", 1)
        if layer["type"] not in _MIXERS:
            raise ValueError(f"layer {index}: unknown mixer type {layer['type']!r} (known: {_MIXERS})")
        mixer = AttentionMixer if layer["type"] == "attention" else ParallelMixer
        self.norm1, self.hc1 = OffsetRMSNorm(width, eps, 0.0), HyperConnection(streams)
        self.mix = mixer(width, layer["mixer"], eps, dtype, linear_method)
        self.mlp = self.norm2 = self.hc2 = None
        if layer.get("mlp") is not None:
            self.norm2, self.hc2 = OffsetRMSNorm(width, eps, 0.0), HyperConnection(streams)
            self.mlp = _feed_forward(width, layer["mlp"], index, dtype, linear_method)


class VufasunForCausalLM(nn.Module):
    uses_ragged_steps = True            # the runner lays every step out as a ragged batch
    supports_float32 = True

    def __init__(self, cfg: dict, dtype: torch.dtype, linear_method: Optional[LinearMethodBase] = None) -> None:
        super().__init__()
        if get_tensor_model_parallel_world_size() != 1:
            raise NotImplementedError("Vufasun layers keep a per-sequence state on one GPU: tensor parallelism is not built for them")
        if linear_method is not None:
            raise NotImplementedError("Vufasun checkpoints are dense: no quantised linear method")
        self.config, self.dtype = cfg, dtype
        self.streams = cfg.get("streams", 1)
        self.runs = [i for i, _ in layer_runs(cfg)]
        self.embed_tokens = VocabParallelEmbedding(cfg["vocab"], cfg["width"], dtype)
        self.layers = nn.ModuleList([VufasunLayer(cfg, i, dtype, None) for i in range(len(cfg["layers"]))])
        self.norm = OffsetRMSNorm(cfg["width"], cfg["norm"]["eps"], 0.0)
        # what the last norm reads: the plain sum of the streams
        self.register_buffer("sum_reads", torch.ones(self.streams, dtype=torch.float32), persistent=False)
        self.sampler = Sampler(cfg["vocab"])
        # set by a caller that wants the sum of the streams after every layer run (a debugging aid; costs a pass per run)
        self.keep_residuals: Optional[list] = None

    # ------------------------------------------------------------------ caches
    @staticmethod
    def cache_layout(cfg: dict, block_size: int) -> List[dict]:
        """Per layer run {"paged": [keys, values], "state": [retention's state, fp32] (parallel layers)}."""
        out = []
        for i, _ in layer_runs(cfg):
            layer = cfg["layers"][i]
            if layer["type"] not in _MIXERS:
                raise ValueError(f"layer {i}: unknown mixer type {layer['type']!r} (known: {_MIXERS})")
            _, g, d, dv = _sizes(_attention_of(layer))
            spec = {"paged": [(block_size, g * d), (block_size, g * dv)]}
            if layer["type"] == "parallel":
                h, _, d, dv = _sizes(layer["mixer"]["right"])
                spec["state"] = [(h, d, dv)]
            out.append(spec)
        return out

    # ----------------------------------------------------------------- forward
    def forward(self, input_ids, positions, kv_caches, input_metadata: InputMetadata):
        if input_metadata.ragged is None:
            raise RuntimeError("Vufasun steps need the ragged layout (InputMetadata.ragged)")
        positions, ids = positions.reshape(-1), input_ids.reshape(-1)
        origin = (ids, self.embed_tokens.weight)
        # (connection, norm of what it reads, its sublayer, run of a mixer or None, last of a layer run?), in order
        path = []
        for r, i in enumerate(self.runs):
            layer = self.layers[i]
            path.append((layer.hc1, layer.norm1, layer.mix, r, layer.mlp is None))
            if layer.mlp is not None:
                path.append((layer.hc2, layer.norm2, layer.mlp, None, True))
        following = [(hc.reads.data, norm) for hc, norm, _, _, _ in path] + [(self.sum_reads, self.norm)]
        h = HyperConnection.begin(origin, *following[0])
        x = torch.empty(ids.numel(), self.streams, self.config["width"], dtype=torch.float32, device=ids.device)
        for s, (hc, _, sublayer, run, last) in enumerate(path):
            y = sublayer(h) if run is None else sublayer(h, positions, kv_caches[run], input_metadata)
            h = hc.step(x, *following[s + 1], self.dtype, origin=origin if s == 0 else None, **y)
            if last and self.keep_residuals is not None:
                self.keep_residuals.append(x.sum(1))
        return h

    def sample(self, hidden_states, sampling_metadata: SamplingMetadata):
        return self.sampler(self.embed_tokens.weight, hidden_states, sampling_metadata)

    def compute_logits(self, hidden_rows: torch.Tensor) -> torch.Tensor:
        """fp32 logits of the given rows of ``forward``'s result: products accumulated and kept in fp32."""
        w = self.embed_tokens.weight
        if hidden_rows.dtype == torch.float32:
            return torch.mm(hidden_rows, w.t())
        return torch.mm(hidden_rows, w.t(), out_dtype=torch.float32)

    # ----------------------------------------------------------------- weights
    @torch.no_grad()
    def finish_random_init(self, seed: int) -> None:
        """After the loader's generic random values (no checkpoint): norm weights, stream connections, sinks and routers of a
        working model's size."""
        g = torch.Generator(device="cpu").manual_seed(seed)

        def rnd(t: torch.Tensor, scale: float, mean: float = 0.0) -> None:
            t.data.copy_(mean + scale * torch.randn(t.shape, generator=g))
        s = self.streams
        for layer in self.layers:
            for norm, hc in ((layer.norm1, layer.hc1), (layer.norm2, layer.hc2)):
                if norm is not None:
                    rnd(norm.weight, 0.1, 1.0)
                    rnd(hc.reads, 0.3 / s, 1.0 / s)
                    rnd(hc.writes, 0.2, 1.0)
                    hc.mix.data.copy_(0.9 * torch.eye(s) + 0.1 / s + 0.05 * torch.randn(s, s, generator=g))
            layer.mix.random_init(rnd)
            if isinstance(layer.mlp, ExpertFeedForward):
                rnd(layer.mlp.experts.router, self.config["width"] ** -0.5)
                layer.mlp.experts.correction.data.zero_()
        rnd(self.norm.weight, 0.1, 1.0)

    def load_weights(self, state: Dict[str, torch.Tensor]) -> None:
        """``state``: checkpoint tensors by name ('embed', 'l<i>.norm1', 'l<i>.norm2', 'l<i>.hc1.*', 'l<i>.hc2.*',
        'l<i>.mix.*', 'l<i>.mlp.*', 'final.norm'); the logits reuse the embedding table."""
        def cast(t):
            return t.to(self.dtype) if t.dtype.is_floating_point else t
        self.embed_tokens.weight.data.copy_(cast(state["embed"]))
        self.norm.weight.data.copy_(state["final.norm"].float())
        for i, layer in enumerate(self.layers):
            pre = f"l{i}."

            def sub(part):
                # norm weights and sinks stay as stored: their layers keep them in fp32
                at = len(pre + part)
                return {k[at:]: (v if k.endswith((".norm", ".sink", ".out")) else cast(v)) for k, v in state.items()
                        if k.startswith(pre + part)}
            layer.mix.load_named(sub("mix."))
            if layer.mlp is not None:
                layer.mlp.load_named(sub("mlp."))
            for norm, hc, q in ((layer.norm1, layer.hc1, "1"), (layer.norm2, layer.hc2, "2")):
                if norm is not None:
                    norm.weight.data.copy_(state[f"{pre}norm{q}"].float())
                    if "streams" in self.config:
                        hc.load_named(state, f"{pre}hc{q}")
