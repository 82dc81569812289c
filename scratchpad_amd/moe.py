"""Mixture-of-experts feed-forward over the HIP kernels of csrc/moe.hip: an fp32 router (sigmoid or softmax scores, a choice
correction, optional group-limited choice), the step's (token, expert) pairs ordered by expert on the device, two grouped
matrix products around the experts' activation, and the weighted sum of each token's experts in a fixed order."""
from typing import NamedTuple, Optional

import torch
from torch import nn

from . import _native
from .layers import ReluSquareFF


class GroupLimitedRouter(nn.Module):
    """ids, weights = top-`top` experts by sigmoid(W x) + correction (weights: the sigmoid without it, not renormalised);
    with `groups` > 1 only experts of the `keep` groups with the largest sum of their two best choices compete."""

    def __init__(self, width: int, experts: int, top: int, groups: int = 1, keep: int = 1):
        super().__init__()
        self.experts, self.top, self.groups, self.keep = experts, top, groups, keep
        self.weight = nn.Parameter(torch.zeros(experts, width, dtype=torch.float32), requires_grad=False)
        self.correction = nn.Parameter(torch.zeros(experts, dtype=torch.float32), requires_grad=False)

    def forward(self, x: torch.Tensor):
        return _native.moe_route(x, self.weight.data, self.correction.data, self.top, self.groups, self.keep)


class ClampedGluExperts(nn.Module):
    """Experts y = W_down (g * sigmoid(alpha g) * (u + 1)), g = min(W_gate x, limit), u = clamp(W_up x, +-limit);
    gate_up [E, 2 ff, W] holds each expert's gate rows, then its up rows."""

    def __init__(self, width: int, experts: int, ff: int, limit: float, alpha: float = 1.702, dtype=None):
        super().__init__()
        self.experts, self.ff, self.limit, self.alpha = experts, ff, limit, alpha
        self.gate_up = nn.Parameter(torch.empty(experts, 2 * ff, width, dtype=dtype), requires_grad=False)
        self.down = nn.Parameter(torch.empty(experts, width, ff, dtype=dtype), requires_grad=False)

    def activation(self, gu: torch.Tensor) -> torch.Tensor:
        return _native.moe_glu(gu, self.limit, self.alpha)

    def forward(self, x: torch.Tensor, ids: torch.Tensor, weights: torch.Tensor) -> torch.Tensor:
        top = ids.shape[1]
        pairs = ids.numel()
        offsets, order, place = _native.moe_align(ids, self.experts)
        gu = _native.moe_grouped_gemm(x, self.gate_up.data, offsets, pairs, order, top)
        y = self.activation(gu)
        z = _native.moe_grouped_gemm(y, self.down.data, offsets, pairs)
        return _native.moe_combine(z, place, weights)


class SparseMoE(nn.Module):
    def __init__(self, width: int, experts: int, top: int, ff: int, limit: float, groups: int = 1, keep: int = 1,
                 dtype=None):
        super().__init__()
        self.router = GroupLimitedRouter(width, experts, top, groups, keep)
        self.experts = ClampedGluExperts(width, experts, ff, limit, dtype=dtype)

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        ids, weights = self.router(x)
        return self.experts(x, ids, weights)


class SoftmaxRouter(nn.Module):
    """ids, weights = the `top` experts with the largest softmax(W x) over ALL experts (fp32 logits); the weights are
    those scores times `scale`, not renormalised over the chosen ones.  ``bias``: the logits are W x + b.  ``renorm``:
    the weights are the softmax over the CHOSEN logits only (they sum to `scale`).  ``correction``: a learned number per
    expert joins its score for the choice, not for the weight.  ``groups`` > ``keep``: the experts form equal groups of
    neighbours and only those of the ``keep`` groups with the largest single choice score compete.  ``gate_row``: one more
    row of ``weight`` (the last) gives a gate per token, sigmoid(w x), returned as a third result."""

    def __init__(self, width: int, experts: int, top: int, scale: float = 1.0, bias: bool = False, renorm: bool = False,
                 correction: bool = False, groups: int = 1, keep: int = 1, gate_row: bool = False):
        super().__init__()
        if experts % groups or not 1 <= keep <= groups or top > keep * (experts // groups):
            raise ValueError("experts must divide into groups, and the kept groups must hold `top` experts")
        self.experts, self.top, self.scale, self.renorm = experts, top, scale, renorm
        self.groups, self.keep, self.gate_row = groups, keep, gate_row
        f32 = dict(dtype=torch.float32)
        self.weight = nn.Parameter(torch.zeros(experts + int(gate_row), width, **f32), requires_grad=False)
        self.bias = nn.Parameter(torch.zeros(experts + int(gate_row), **f32), requires_grad=False) if bias else None
        self.correction = nn.Parameter(torch.zeros(experts, **f32), requires_grad=False) if correction else None

    def forward(self, x: torch.Tensor):
        return _native.moe_route_softmax(x, self.weight.data, self.top, self.scale,
                                         None if self.bias is None else self.bias.data, self.renorm,
                                         None if self.correction is None else self.correction.data, self.groups, self.keep,
                                         self.gate_row)


class SiluGluExperts(ClampedGluExperts):
    """Experts y = W_down (silu(W_gate x) * (W_up x)): the same stacked layout and grouped products, no clamps."""

    def __init__(self, width: int, experts: int, ff: int, dtype=None):
        super().__init__(width, experts, ff, 0.0, dtype=dtype)

    def activation(self, gu: torch.Tensor) -> torch.Tensor:
        return _native.silu_and_mul(gu)


class SoftmaxMoE(nn.Module):
    """SoftmaxRouter + SiluGluExperts; `forward` returns the routed experts' weighted sum (a shared expert, if the model
    has one, is a dense feed-forward of its own beside this)."""

    def __init__(self, width: int, experts: int, top: int, ff: int, scale: float = 1.0, dtype=None):
        super().__init__()
        self.router = SoftmaxRouter(width, experts, top, scale)
        self.experts = SiluGluExperts(width, experts, ff, dtype=dtype)

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        ids, weights = self.router(x)
        return self.experts(x, ids, weights)


class ChosenSoftmaxMoE(nn.Module):
    """Experts chosen by the largest router logits W x + b and weighted by the softmax over the chosen logits only, each a
    clamped gated unit (ClampedGluExperts); `forward` returns their weighted sum."""

    def __init__(self, width: int, experts: int, top: int, ff: int, limit: float, dtype=None):
        super().__init__()
        self.router = SoftmaxRouter(width, experts, top, bias=True, renorm=True)
        self.experts = ClampedGluExperts(width, experts, ff, limit, dtype=dtype)

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        ids, weights = self.router(x)
        return self.experts(x, ids, weights)


class ReluSquareExperts(nn.Module):
    """Experts y = W_down max(W_up x, 0)^2, stacked: up [E, ff, W], down [E, W, ff].  ``rows`` returns the chosen experts'
    outputs in the pairs' order by expert, not yet weighted; pairs whose id is E or more (outputs of the router that stand
    for no expert of this module) are left out of both products and their rows are undefined."""

    def __init__(self, width: int, experts: int, ff: int, dtype=None):
        super().__init__()
        self.experts, self.ff = experts, ff
        self.up = nn.Parameter(torch.empty(experts, ff, width, dtype=dtype), requires_grad=False)
        self.down = nn.Parameter(torch.empty(experts, width, ff, dtype=dtype), requires_grad=False)

    def put(self, e: int, up: torch.Tensor, down: torch.Tensor) -> None:
        """expert e's matrices into the stacks"""
        for stack, value in ((self.up, up), (self.down, down)):
            if value.shape != stack.shape[1:]:
                raise RuntimeError(f"shape {tuple(value.shape)} does not fit an expert's {tuple(stack.shape[1:])}")
            stack.data[e].copy_(value.to(stack.dtype))

    def rows(self, x: torch.Tensor, ids: torch.Tensor, outputs: Optional[int] = None):
        """(z [T * top, W], place int32 [T * top]): pair p's output is z[place[p]].  ``outputs``: how many different ids there
        are (default: the experts)"""
        offsets, order, place = _native.moe_align(ids, outputs or self.experts)
        y = _native.moe_grouped_gemm(x, self.up.data, offsets, ids.numel(), order, ids.shape[1], act="relu2")
        return _native.moe_grouped_gemm(y, self.down.data, offsets, ids.numel()), place


class MixtureRows(NamedTuple):
    """A mixture's result before its sum, for whoever joins it to the stream (layers.PostNorm): per token
    sum_k weights[t, k] (z[place[t, k]], or the layer's input where ids[t, k] >= experts) + gate[t] dense[t]"""
    z: torch.Tensor
    ids: torch.Tensor
    place: torch.Tensor
    weights: torch.Tensor
    experts: int
    dense: Optional[torch.Tensor] = None
    gate: Optional[torch.Tensor] = None


class IdentityMoE(nn.Module):
    """Experts and identity experts under one softmax router: the last ``identity`` of the router's outputs stand for experts
    that hand their input on.  Weighted by their scores over ALL outputs (not renormalised), chosen by score plus a learned
    correction within the best groups (SoftmaxRouter).  ``shared_ff``: a further expert of that width runs for every token,
    its result times sigmoid(w x); that gate's row rides in the router's fp32 product.  ``forward`` returns MixtureRows."""

    def __init__(self, width: int, experts: int, identity: int, top: int, ff: int, groups: int = 1, keep: int = 1,
                 shared_ff: Optional[int] = None, dtype=None):
        super().__init__()
        self.outputs = experts + identity
        self.router = SoftmaxRouter(width, self.outputs, top, correction=True, groups=groups, keep=keep,
                                    gate_row=shared_ff is not None)
        self.experts = ReluSquareExperts(width, experts, ff, dtype)
        self.shared = ReluSquareFF(width, shared_ff, dtype=dtype) if shared_ff is not None else None

    def forward(self, h: torch.Tensor, x: torch.Tensor) -> MixtureRows:
        """h: the layer's input in the experts' dtype; x: the same in fp32, which the router reads"""
        ids, weights, *gate = self.router(x)
        z, place = self.experts.rows(h, ids, self.outputs)
        if self.shared is None:
            return MixtureRows(z, ids, place, weights, self.experts.experts)
        return MixtureRows(z, ids, place, weights, self.experts.experts, self.shared(h), gate[0])
