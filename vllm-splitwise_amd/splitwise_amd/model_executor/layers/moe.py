"""Mixture-of-experts feed-forward layers.

``TableRoutedExperts``: no learned router -- a table [vocab, top] names each token id's experts, every chosen
expert weighs 1 / top.  An expert is down(gelu(up x)) with the exact (erf) gelu and no biases.  An optional
shared expert of the same form runs for every token and is added after a per-token sigmoid gate.

``GroupRoutedExperts``: a learned sigmoid router in fp32 with a selection bias that enters the choice but not the
weights, a choice limited to the best groups of neighbouring experts, weights normalised over the chosen experts
and scaled; an expert is down(relu(up x)^2); an optional shared expert of the same form is returned beside the
routed sum so that the caller's residual add can take both.  The same layer, by its options, is a SOFTMAX router
(``score="softmax"``: scores are the softmax over all experts), whose groups score their best expert
(``group_score="max"``), whose weights are the chosen scores as they are (``normalize=False``) and whose experts have
a gated hidden layer with limits (``activation="clamped_glu"``: g = min(gate x, limit), u = clamp(up x, +-limit),
g sigmoid(alpha g) (u + shift); alpha 1, no limit and shift 0 make it silu(g) u).  ``score="softmax_chosen"``: the choice
goes by the logits and the weights are their softmax over the chosen ones (a ``router_bias`` is part of the logits).
``weigh_input``: an expert's weight multiplies what the expert reads instead of what it returns (the two differ: the
hidden layer is not linear).  A shared expert has the routed experts' form: with a gated hidden layer it is
down(silu(gate x) * up x).

Rows are grouped by expert on the device (a stable sort of the (row, choice) pairs by expert id, then a binary
search for every expert's first pair), so each expert's rows are one contiguous run and the host never waits.
"""
from typing import Dict, Optional, Tuple

import torch
import torch.nn as nn
import torch.nn.functional as F

from ... import _C
from .basic import GatedActivation, ReluSquared
from .linear import ColumnParallelLinear, MergedColumnParallelLinear, RowParallelLinear


class TableRoutedExperts(nn.Module):
    def __init__(self, width: int, vocab: int, num_experts: int, top: int, ff: int, shared_ff: Optional[int],
                 dtype: torch.dtype, linear_method=None) -> None:
        super().__init__()
        self.width, self.num_experts, self.top, self.ff = width, num_experts, top, ff
        self.table = nn.Parameter(torch.zeros(vocab, top, dtype=torch.int32), requires_grad=False)
        self.up = nn.Parameter(torch.empty(num_experts, ff, width, dtype=dtype), requires_grad=False)
        self.down = nn.Parameter(torch.empty(num_experts, width, ff, dtype=dtype), requires_grad=False)
        self.shared_ff = shared_ff
        if shared_ff:
            # shared expert's up projection and its gate read the same input: one GEMM
            self.shared_in = MergedColumnParallelLinear(width, [shared_ff, 1], False, dtype, linear_method)
            self.shared_down = RowParallelLinear(shared_ff, width, False, dtype, linear_method)

    def route(self, token_ids: torch.Tensor):
        """-> (order [rows * top] int32: pair index row * top + choice, sorted by expert;
               expert_start [experts + 1] int32)."""
        experts = self.table.data.index_select(0, token_ids).view(-1)              # [rows * top]
        by_expert, order = torch.sort(experts, stable=True)
        # first sorted pair of every expert: no count ever travels to the host
        edges = torch.arange(self.num_experts + 1, dtype=experts.dtype, device=experts.device)
        start = torch.searchsorted(by_expert, edges).to(torch.int32)
        return order.to(torch.int32), start

    def forward(self, h: torch.Tensor, token_ids: torch.Tensor) -> torch.Tensor:
        """-> fp32 [rows, width]: the experts' sum is accumulated in fp32."""
        rows = h.shape[0]
        order, start = self.route(token_ids)
        out = torch.zeros(rows, self.width, dtype=torch.float32, device=h.device)
        _C.mixer_ops.expert_ffn(out, h, self.up.data, self.down.data, order, start, self.top, 1.0 / self.top)
        if self.shared_ff:
            both = self.shared_in(h)
            hidden = F.gelu(both[:, :self.shared_ff])
            shared = self.shared_down(hidden)
            out.addcmul_(torch.sigmoid(both[:, self.shared_ff:].float()), shared.float())
        return out

    def load_named(self, w: Dict[str, torch.Tensor]) -> None:
        self.table.data.copy_(w["table"].to(torch.int32))
        self.up.data.copy_(torch.stack([w[f"e{e}.up"] for e in range(self.num_experts)]))
        self.down.data.copy_(torch.stack([w[f"e{e}.down"] for e in range(self.num_experts)]))
        if self.shared_ff:
            self.shared_in.weight.data.copy_(torch.cat([w["shared.up"], w["shared.sg"]], 0))
            self.shared_down.weight.data.copy_(w["shared.down"])


def group_pairs_by_expert(experts: torch.Tensor, num_experts: int):
    """experts int32 [rows, top] -> (order int32 [rows * top]: pair indices row * top + choice grouped by expert,
    expert_start int32 [experts + 1]); one launch on the device."""
    return _C.mixer_ops.group_pairs(experts, num_experts)


class GroupRoutedExperts(nn.Module):
    def __init__(self, width: int, num_experts: int, top: int, ff: int, shared_ff: Optional[int], groups: int,
                 keep_groups: int, scale: float, dtype: torch.dtype, linear_method=None, score: str = "sigmoid",
                 group_score: str = "top2", normalize: bool = True, activation: str = "relu2",
                 limit: float = float("inf"), glu_alpha: float = 1.702, glu_shift: float = 1.0, router_bias: bool = False,
                 router_dtype: torch.dtype = torch.float32, weigh_input: bool = False) -> None:
        super().__init__()
        if score not in ("sigmoid", "softmax", "softmax_chosen") or group_score not in ("top2", "max") or \
                activation not in ("relu2", "clamped_glu"):
            raise ValueError(f"unknown router score {score!r}, group score {group_score!r} or activation {activation!r}")
        if activation == "clamped_glu" and shared_ff and (glu_alpha, limit, glu_shift) != (1.0, float("inf"), 0.0):
            raise NotImplementedError("a shared expert whose gated hidden layer is not silu(gate) * up")
        self.weigh_input = bool(weigh_input)
        self.softmax = {"sigmoid": 0, "softmax": _C.mixer_ops.ROUTER_SOFTMAX,
                        "softmax_chosen": _C.mixer_ops.ROUTER_SOFTMAX_CHOSEN}[score]
        self.group_best_one, self.normalize = group_score == "max", bool(normalize)
        self.glu = (float(glu_alpha), float(limit), float(glu_shift)) if activation == "clamped_glu" else None
        if num_experts % groups != 0 or not (1 <= keep_groups <= groups) or keep_groups * (num_experts // groups) < top:
            raise ValueError(f"{num_experts} experts in {groups} groups with {keep_groups} kept cannot give {top} choices")
        self.width, self.num_experts, self.top, self.ff = width, num_experts, top, ff
        self.groups, self.keep_groups, self.scale = groups, keep_groups, float(scale)
        # the router's products are fp32 whatever the model's dtype; a checkpoint's bf16 router may be kept as it is
        # (``router_dtype``): its products with bf16 inputs are exact in fp32
        self.router = nn.Parameter(torch.zeros(num_experts, width, dtype=router_dtype), requires_grad=False)
        self.router_bias = nn.Parameter(torch.zeros(num_experts, dtype=torch.float32), requires_grad=False) \
            if router_bias else None
        self.correction = nn.Parameter(torch.zeros(num_experts, dtype=torch.float32), requires_grad=False)
        # a gated hidden layer: gate and up rows in runs of 16, as the fused kernel reads them (``mixer_ops.glu_rows``)
        self.up = nn.Parameter(torch.empty(num_experts, 32 * (-(-ff // 16)) if self.glu else ff, width, dtype=dtype),
                               requires_grad=False)
        self.down = nn.Parameter(torch.empty(num_experts, width, ff, dtype=dtype), requires_grad=False)
        self.shared_ff = shared_ff
        if shared_ff:
            self.shared_up = MergedColumnParallelLinear(width, [shared_ff, shared_ff], False, dtype, linear_method) \
                if self.glu else ColumnParallelLinear(width, shared_ff, False, dtype, linear_method)
            self.shared_act = GatedActivation("silu") if self.glu else ReluSquared()
            self.shared_down = RowParallelLinear(shared_ff, width, False, dtype, linear_method)

    def router_logits(self, h: torch.Tensor) -> torch.Tensor:
        """fp32 [rows, experts]: products and sums in fp32 (the library's GEMM; no reduced-precision matrix mode is switched
        on)."""
        w = self.router.data.t()
        if w.dtype == h.dtype and h.dtype != torch.float32:
            if self.router_bias is None:
                return torch.mm(h, w, out_dtype=torch.float32)
            return torch.addmm(self.router_bias.data, h, w, out_dtype=torch.float32)
        if self.router_bias is None:
            return torch.matmul(h.float(), w)
        return torch.addmm(self.router_bias.data, h.float(), w)

    def forward(self, h: torch.Tensor) -> Tuple[Optional[torch.Tensor], torch.Tensor]:
        """-> (shared expert's output in h's dtype or None, routed experts' weighted sum in fp32)."""
        out = torch.empty(h.shape[0], self.width, dtype=torch.float32, device=h.device)
        chosen, weights = _C.mixer_ops.group_router(self.router_logits(h), self.correction.data, self.top, self.groups,
                                                    self.keep_groups, self.scale, self.softmax, self.group_best_one,
                                                    self.normalize, clear=out)
        order, start = group_pairs_by_expert(chosen, self.num_experts)
        _C.mixer_ops.expert_ffn(out, h, self.up.data, self.down.data, order, start, self.top, 1.0,
                                activation=_C.mixer_ops.ACT_RELU2, pair_weight=weights, glu=self.glu,
                                weigh_input=self.weigh_input)
        shared = None
        if self.shared_ff:
            shared = self.shared_down(self.shared_act(self.shared_up(h)))
        return shared, out

    def load_named(self, w: Dict[str, torch.Tensor]) -> None:
        self.router.data.copy_(w["router"])
        if self.router_bias is not None:
            self.router_bias.data.copy_(w["router.b"].float())
        if "correction" in w:
            self.correction.data.copy_(w["correction"].float())
        if self.glu:
            self.up.data.copy_(_C.mixer_ops.glu_rows(torch.stack([w[f"e{e}.gate"] for e in range(self.num_experts)]),
                                                     torch.stack([w[f"e{e}.up"] for e in range(self.num_experts)])))
        else:
            self.up.data.copy_(torch.stack([w[f"e{e}.up"] for e in range(self.num_experts)]))
        self.down.data.copy_(torch.stack([w[f"e{e}.down"] for e in range(self.num_experts)]))
        if self.shared_ff:
            self.shared_up.weight.data.copy_(torch.cat([w["shared.gate"], w["shared.up"]], 0) if self.glu else w["shared.up"])
            self.shared_down.weight.data.copy_(w["shared.down"])
