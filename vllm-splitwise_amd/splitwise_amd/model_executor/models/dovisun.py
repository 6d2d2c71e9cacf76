"""Dovisun: a decoder whose layers are listed one by one in its config.json, whose two sublayers run side by side on ONE
norm of the stream, and a block of whose layers runs several times in a row with the same weights.

Each entry of ``layers`` names the layer's token mixer -- ``attention`` (grouped query heads without positions, unit
queries and keys, one more term in the softmax's denominator) or ``latent_attention`` (queries through a latent of their
own, keys and values of all heads from one small latent per token plus a rotated key part shared by the heads, YaRN
frequencies, one sigmoid gate per head) -- with the mixer's sizes, and its feed-forward: ``dense`` (down(relu(up h)^2)),
``moe`` (router choice by the biased logits, weights = softmax over the chosen, experts down(silu(gate h) * up h)) or
none.

With N(x) = x / rms(x) * w and x_0 = scale * embedding rows:
    a layer:                h = N(x);  x <- x + (mixer(h) + ff(h))
    ``loop``:               layers start .. stop - 1 run ``times`` times in a row; before the first of them, each time,
                            x <- W_x x + W_0 x_0
    the logits:             cap * tanh(head N(x) / cap)
The stream is fp32.  All projections of a layer's input -- the mixer's and a dense feed-forward's -- are one GEMM, and so
are the two that lead back to the stream: the mixer's heads and the feed-forward's hidden channels are written side by
side into one row.  The add of a layer and the norm of the next are one kernel.
Steps arrive in the ragged layout (``InputMetadata.ragged``): any mix of prompt portions and decoded tokens.

The worker allocates what ``cache_layout`` asks for per layer RUN: a layer that runs several times has pages of its own
for every pass.
"""
from typing import Dict, List, Optional

import torch
import torch.nn as nn

from ... import _C
from ..input_metadata import InputMetadata
from ..layers.attention import LatentQueryAttention, UnitHeadAttention
from ..layers.basic import LoopInput, OffsetRMSNorm, yarn_rotary
from ..layers.linear import LinearMethodBase, MergedColumnParallelLinear, RowParallelLinear
from ..layers.moe import GroupRoutedExperts
from ..layers.sampler import Sampler, SamplingMetadata
from ..layers.vocab_parallel_embedding import VocabParallelEmbedding
from ..parallel_state import get_tensor_model_parallel_world_size
from .layer_list import layer_runs

_MIXERS = ("attention", "latent_attention")
_DEFAULT_Q_RANK_DIVISOR = 4       # of a model without a checkpoint whose config does not name the query latent's size


def normalize_config(raw: dict) -> dict:
    """The engine's generic geometry keys for a Dovisun config.json."""
    cfg = dict(raw)
    cfg["architecture"] = "dovisun"
    cfg["vocab_size"] = raw["vocab"]
    cfg["hidden_size"] = raw["width"]
    cfg["num_hidden_layers"] = len(layer_runs(raw))
    mixers = [l["mixer"] for l in raw["layers"]]
    cfg["num_attention_heads"] = mixers[0]["heads"] if mixers else 1
    cfg["num_key_value_heads"] = mixers[0].get("kv_heads", mixers[0]["heads"]) if mixers else 1
    cfg.setdefault("max_position_embeddings", 1 << 20)       # angles come from fp32 positions: no table to outgrow
    cfg.setdefault("torch_dtype", "bfloat16")
    return cfg


def _q_rank(cfg: dict, m: dict) -> int:
    return int(m.get("q_rank", max(1, cfg["width"] // _DEFAULT_Q_RANK_DIVISOR)))


class DovisunLayer(nn.Module):
    def __init__(self, cfg: dict, index: int, dtype, linear_method) -> None:
        super().__init__()
        layer = cfg["layers"][index]
        width, eps, m, mlp = cfg["width"], cfg["norm"]["eps"], layer["mixer"], layer.get("mlp")
        self.kind = layer["type"]
        self.norm1 = OffsetRMSNorm(width, eps, 0.0)
        h, d = m["heads"], m["dim"]
        dv = m.get("vdim", d)
        # ---- feed-forward
        self.experts, self.ff = None, 0
        if mlp is not None:
            if mlp["kind"] == "dense":
                self.ff = int(mlp["ff"])
            elif mlp["kind"] == "moe":
                r = mlp["router"]
                self.experts = GroupRoutedExperts(width, r["experts"], r["top"], mlp["expert"]["ff"], None, 1, 1, 1.0, dtype,
                                                  linear_method, score="softmax_chosen", activation="clamped_glu",
                                                  glu_alpha=1.0, glu_shift=0.0, router_bias=True, router_dtype=dtype)
            else:
                raise ValueError(f"layer {index}: unknown feed-forward kind {mlp['kind']!r}")
        # ---- mixer; ``names``: the checkpoint's matrices in the order of the input projection's columns
        if self.kind == "attention":
            g = m.get("kv_heads", h)
            self.names, mixer_sizes = ["q", "k", "v"], [h * d, g * d, g * dv]
            self.attn = UnitHeadAttention(h, g, d, dv, m["scale"], eps, sink=True)
        elif self.kind == "latent_attention":
            dr, rank, q_rank = m["rot_dim"], m["kv_rank"], _q_rank(cfg, m)
            rot = m.get("rot") or {"dims": dr, "base": 10000.0}
            if rot["dims"] != dr:
                raise ValueError(f"layer {index}: the whole rotated part turns: rot.dims {rot['dims']} != rot_dim {dr}")
            freqs, amplitude = yarn_rotary(dr, rot["base"], rot.get("scaling"))
            self.names, mixer_sizes = ["dq", "dkv", "g"], [q_rank, rank + dr, h]
            self.attn = LatentQueryAttention(h, d, dr, dv, rank, q_rank, m["scale"], freqs, amplitude, eps, dtype)
        else:
            raise ValueError(f"layer {index}: unknown mixer type {self.kind!r} (known: {_MIXERS})")
        # columns: up | mixer's parts | padding to whole 32-byte runs, so that every row begins on one
        self.heads_size = h * dv
        sizes = ([self.ff] if self.ff else []) + mixer_sizes
        self.pad = -sum(sizes) % 16
        self.sizes = sizes
        self.in_proj = MergedColumnParallelLinear(width, sizes + ([self.pad] if self.pad else []), False, dtype, linear_method)
        self.out_proj = RowParallelLinear(self.ff + self.heads_size, width, False, dtype, linear_method)

    def forward(self, h: torch.Tensor, positions: torch.Tensor, cache: List[torch.Tensor], md: InputMetadata):
        """h: the layer's norm of the stream.  -> the addends of the stream: (the mixer's output, with the dense
        feed-forward's in it, in the activation dtype; the experts' sum in fp32 or None)."""
        proj = self.in_proj(h)
        cols, lo = [], 0
        for n in self.sizes:
            cols.append(proj[:, lo:lo + n])
            lo += n
        # hidden channels | heads: one row of the output projection's input
        both = torch.empty(h.shape[0], self.ff + self.heads_size, dtype=h.dtype, device=h.device)
        if self.ff:
            _C.mixer_ops.relu2(both[:, :self.ff], cols.pop(0))
        heads = both[:, self.ff:]
        if self.kind == "attention":
            self.attn(cols[0], cols[1], cols[2], cache[0], cache[1], md, heads)
        else:
            self.attn(cols[0], cols[1], cols[2], positions, cache[0], md, heads)
        routed = self.experts(h)[1] if self.experts is not None else None
        return self.out_proj(both), routed

    def load_named(self, mix: Dict[str, torch.Tensor], mlp: Dict[str, torch.Tensor]) -> None:
        parts = ([mlp["up"]] if self.ff else []) + [mix[n] for n in self.names]
        self.in_proj.weight.data.zero_()                       # the padding's rows
        self.in_proj.weight.data[:sum(self.sizes)].copy_(torch.cat(parts, 0))
        self.out_proj.weight.data.copy_(torch.cat(([mlp["down"]] if self.ff else []) + [mix["o"]], 1))
        if self.kind == "latent_attention":
            self.attn.query_norm.data.copy_(mix["dq.norm"].float())
            self.attn.latent_norm.data.copy_(mix["dkv.norm"].float())
            self.attn.load_up_projections(mix["uq"], mix["uk"], mix["uv"])
        if self.experts is not None:
            self.experts.load_named(mlp)


class DovisunForCausalLM(nn.Module):
    uses_ragged_steps = True            # the runner lays every step out as a ragged batch
    supports_float32 = True

    def __init__(self, cfg: dict, dtype: torch.dtype, linear_method: Optional[LinearMethodBase] = None) -> None:
        super().__init__()
        if get_tensor_model_parallel_world_size() != 1:
            raise NotImplementedError("Dovisun layers are laid out for one GPU: tensor parallelism is not built for them")
        if linear_method is not None:
            raise NotImplementedError("Dovisun checkpoints are dense: no quantised linear method")
        self.config, self.dtype = cfg, dtype
        width, eps = cfg["width"], cfg["norm"]["eps"]
        self.embed_scale = float((cfg.get("embedding") or {}).get("scale", 1.0))
        self.runs = layer_runs(cfg)
        self.embed_tokens = VocabParallelEmbedding(cfg["vocab"], width, dtype)
        self.layers = nn.ModuleList([DovisunLayer(cfg, i, dtype, None) for i in range(len(cfg["layers"]))])
        self.loop_in = LoopInput(width, self.embed_scale, dtype) if cfg.get("loop") else None
        self.norm = OffsetRMSNorm(width, eps, 0.0)
        self.head = nn.Parameter(torch.zeros(cfg["vocab"], width, dtype=dtype), requires_grad=False)
        self.sampler = Sampler(cfg["vocab"], logit_softcap=cfg.get("logit_softcap"))
        # set by a caller that wants the stream after every layer run (a debugging aid; costs a copy per run)
        self.keep_residuals: Optional[list] = None

    # ------------------------------------------------------------------ caches
    @staticmethod
    def note_tensor_shapes(cfg: dict, shapes: Dict[str, tuple]) -> None:
        """The query latent's size, where config.json does not name it, is a tensor's shape."""
        for i, layer in enumerate(cfg["layers"]):
            name = f"l{i}.mix.dq"
            if layer["type"] == "latent_attention" and name in shapes:
                layer["mixer"].setdefault("q_rank", int(shapes[name][0]))

    @staticmethod
    def cache_layout(cfg: dict, block_size: int) -> List[dict]:
        """Per layer run {"paged": [shape per page, ...]}: keys and values of an attention layer, the one row of latent and
        shared key part of a latent-attention layer."""
        out = []
        for i, _ in layer_runs(cfg):
            layer = cfg["layers"][i]
            m = layer["mixer"]
            if layer["type"] == "attention":
                g = m.get("kv_heads", m["heads"])
                out.append({"paged": [(block_size, g * m["dim"]), (block_size, g * m.get("vdim", m["dim"]))]})
            elif layer["type"] == "latent_attention":
                out.append({"paged": [(block_size, m["kv_rank"] + m["rot_dim"])]})
            else:
                raise ValueError(f"layer {i}: unknown mixer type {layer['type']!r} (known: {_MIXERS})")
        return out

    # ----------------------------------------------------------------- forward
    def forward(self, input_ids, positions, kv_caches, input_metadata: InputMetadata):
        if input_metadata.ragged is None:
            raise RuntimeError("Dovisun steps need the ragged layout (InputMetadata.ragged)")
        positions = positions.reshape(-1)
        ids = input_ids.reshape(-1)
        new = lambda dtype: torch.empty(ids.numel(), self.config["width"], dtype=dtype, device=ids.device)   # noqa: E731
        x = new(torch.float32)
        loop, n = self.loop_in, len(self.runs)
        rows = new(self.dtype) if loop is not None else None
        first = self._norm_of_run(0)
        h = None
        if n and self.runs[0][1]:                              # a pass begins at once: its input is what gets normed
            _C.mixer_ops.embed_stream(x, ids, self.embed_tokens.weight, self.embed_scale, rows)
        else:
            h = new(self.dtype)
            _C.mixer_ops.embed_stream(x, ids, self.embed_tokens.weight, self.embed_scale, rows, first.weight.data,
                                      first.offset, first.variance_epsilon, h)
        from_embedding = loop.start(rows) if loop is not None else None
        if h is None:
            x = loop(x)
            h = first.add_norm(x, self.dtype, None, None, from_embedding)
        for r, (i, _) in enumerate(self.runs):
            a, c = self.layers[i](h, positions, kv_caches[r], input_metadata)
            nxt = self._norm_of_run(r + 1)
            if r + 1 < n and self.runs[r + 1][1]:              # the next run begins a pass
                x_new = loop(x, a, None, c)                    # x += a + c;  x_new = W_x x
                if self.keep_residuals is not None:
                    self.keep_residuals.append(x.clone())
                x = x_new
                h = nxt.add_norm(x, self.dtype, None, None, from_embedding)      # the pass's input and its norm
                continue
            h = nxt.add_norm(x, self.dtype, a, None, c)        # x += a + c;  h = the next norm of x
            if self.keep_residuals is not None:
                self.keep_residuals.append(x.clone())
        return h

    def _norm_of_run(self, r: int) -> OffsetRMSNorm:
        return self.layers[self.runs[r][0]].norm1 if r < len(self.runs) else self.norm

    def sample(self, hidden_states, sampling_metadata: SamplingMetadata):
        return self.sampler(self.head, hidden_states, sampling_metadata)

    def compute_logits(self, hidden_rows: torch.Tensor) -> torch.Tensor:
        """fp32 logits of the given rows of ``forward``'s result: products accumulated and kept in fp32."""
        if hidden_rows.dtype == torch.float32:
            logits = torch.mm(hidden_rows, self.head.t())
        else:
            logits = torch.mm(hidden_rows, self.head.t(), out_dtype=torch.float32)
        return self.sampler.cap_logits(logits)

    # ----------------------------------------------------------------- weights
    @torch.no_grad()
    def finish_random_init(self, seed: int) -> None:
        """After the loader's generic random values (no checkpoint): norm weights and routers of a working model's size."""
        g = torch.Generator(device="cpu").manual_seed(seed)

        def rnd(t: torch.Tensor, scale: float, mean: float = 0.0) -> None:
            t.data.copy_(mean + scale * torch.randn(t.shape, generator=g))
        if self.loop_in is not None:                           # the two halves of the stream share one matrix
            self.loop_in.load(torch.cat([self.loop_in.stream_weight.data[:, :self.config["width"]],
                                         self.loop_in.embed_weight.data], 1))
        for layer in self.layers:
            rnd(layer.norm1.weight, 0.1, 1.0)
            if layer.kind == "latent_attention":
                layer.attn.query_norm.data.fill_(1.0)
                layer.attn.latent_norm.data.fill_(1.0)
            if layer.experts is not None:
                rnd(layer.experts.router, layer.experts.width ** -0.5)
                rnd(layer.experts.router_bias, 0.1)
                layer.experts.correction.data.zero_()
        rnd(self.norm.weight, 0.1, 1.0)

    def load_weights(self, state: Dict[str, torch.Tensor]) -> None:
        """``state``: checkpoint tensors by name ('embed', 'loop.in', 'l<i>.norm1', 'l<i>.mix.*', 'l<i>.mlp.*', 'final.norm',
        'head')."""
        def cast(t):
            return t.to(self.dtype) if t.dtype.is_floating_point else t
        self.embed_tokens.weight.data.copy_(cast(state["embed"]))
        self.head.data.copy_(cast(state["head"]))
        self.norm.weight.data.copy_(state["final.norm"].float())
        if self.loop_in is not None:
            self.loop_in.load(cast(state["loop.in"]))
        for i, layer in enumerate(self.layers):
            pre = f"l{i}."
            layer.norm1.weight.data.copy_(state[pre + "norm1"].float())

            def sub(part):
                # router biases and norm weights stay as stored: their layers keep them in fp32
                at = len(pre + part)
                return {k[at:]: (v if k.endswith((".norm", "router.b")) else cast(v)) for k, v in state.items()
                        if k.startswith(pre + part)}
            layer.load_named(sub("mix."), sub("mlp."))
