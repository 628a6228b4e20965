"""Mixture-of-experts feed-forward for layer-spec models.

Router: softmax over all experts in fp32, the ``top`` largest scores renormalised and scaled, or
sigmoid scores taken as they are, or the ``top`` largest logits (with a bias) and a softmax over those
alone (``ops.seqmix.moe_route``), or softmax scores that are corrected and limited to groups of experts for the
choice only (``ops.seqmix.moe_route_grouped``).  Experts: clamped or plain silu
gated-linear units or squared-ReLU units without a gate (then ``w_gu`` is [E, ff, W]), the router's weight on their output or on their input, weights stacked per layer as
``w_gu`` [E, 2 ff, W] (gate rows, then up rows) and ``w_down`` [E, W, ff]; decode-sized steps read
only the chosen experts' rows, prompt-sized steps sort (token, choice) pairs by expert
(``ops.seqmix.moe_experts``).  The shared expert is a dense unit of the same form.  ``forward``
returns the shared expert's output and the chosen experts' outputs with their weights apart: the
layer's output norm adds them up in fp32 in one kernel with the residual add.  ``run`` also returns the
shared expert's weight per token and leaves prompt-sized steps' rows sorted by expert, for a residual kernel
that takes both.
"""
from __future__ import annotations

from typing import NamedTuple, Optional

import torch
import torch.nn as nn

from ..ops import seqmix
from .configs import MoESpec
from .layers import Linear


class MoEOut(NamedTuple):
    shared: Optional[torch.Tensor]      # the shared expert's output [T, W]
    shared_w: Optional[torch.Tensor]    # its weight fp32 [T] (None: 1)
    parts: torch.Tensor                 # the chosen experts' outputs [T, top, W]
    wts: Optional[torch.Tensor]         # their weights fp32 [T, top]
    rows: Optional[torch.Tensor]        # int32 [T, top]: each choice's row of parts viewed [-1, W] (None: in order)


class MoEFeedForward(nn.Module):
    def __init__(self, spec: MoESpec, width: int, dtype, device):
        super().__init__()
        self.spec = spec
        s = spec
        # a shared expert's gate is one more row of the router
        self.router = nn.Parameter(torch.zeros(s.experts + int(s.shared_gate), width, dtype=torch.float32, device=device), requires_grad=False)
        self.router_b = nn.Parameter(torch.zeros(s.experts, dtype=torch.float32, device=device), requires_grad=False) \
            if s.router_bias else None
        self.correction = nn.Parameter(torch.zeros(s.experts, dtype=torch.float32, device=device), requires_grad=False) \
            if s.correction else None
        up = 2 if s.glu else 1
        self.w_gu = nn.Parameter(torch.zeros(s.experts, up * s.ff, width, dtype=dtype, device=device), requires_grad=False)
        self.w_down = nn.Parameter(torch.zeros(s.experts, width, s.ff, dtype=dtype, device=device), requires_grad=False)
        if s.shared_ff:
            self.shared_gu = Linear(width, up * s.shared_ff, False, dtype, device)
            self.shared_down = Linear(s.shared_ff, width, False, dtype, device)

    def forward(self, h: torch.Tensor):
        """h [T, W] -> (shared expert's output [T, W] or None, expert outputs [T, top, W], weights fp32
        [T, top] still to be applied to them, or None when the experts ran on weighted inputs)."""
        s = self.spec
        idx, wts = seqmix.moe_route(h, self.router, s.top, s.scale, s.router, self.router_b)
        on_input = s.weight_on == "input"
        parts = seqmix.moe_experts(h, idx, self.w_gu, self.w_down, s.limit, s.act, wts if on_input else None)
        if on_input:
            wts = None
        shared = None
        if s.shared_ff:
            shared = self.shared_down(seqmix.glu_clamp(self.shared_gu(h), s.shared_ff, s.shared_limit))
        return shared, parts, wts

    def run(self, h: torch.Tensor) -> MoEOut:
        """The form with a grouped choice (squared-ReLU or silu-gated experts): h [T, W] -> MoEOut."""
        s = self.spec
        assert s.router == "softmax" and s.weight_on == "output" and (s.act == "relu2" or (s.act == "silu_glu" and not s.shared_ff))
        idx, wts, shared_w = seqmix.moe_route_grouped(h, self.router, s.top, s.scale, self.correction, s.groups, s.groups_keep,
                                                      s.shared_gate)
        if s.shared_ff and h.shape[0] < seqmix.MOE_GEMM_MIN:
            parts, shared = seqmix.moe_experts_shared(h, idx, self.w_gu, self.w_down, self.shared_gu.weight,
                                                      self.shared_down.weight)
            return MoEOut(shared, shared_w, parts, wts, None)
        parts, rows = seqmix.moe_experts(h, idx, self.w_gu, self.w_down, 0.0, s.act, sorted_rows=True)
        shared = self.shared_down(seqmix.relu2(self.shared_gu(h))) if s.shared_ff else None
        return MoEOut(shared, shared_w, parts, wts, rows)
