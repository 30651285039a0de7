"""A mixture of small feed-forward experts with a router, and optionally one shared expert ("moe").

  z = W_r h + b                       router logits, in 32-bit
  the ``top`` largest logits are chosen; their weights are the soft-max over the chosen logits alone
  (``score`` = "sigmoid": s = sigmoid(z); the choice goes by s + correction, inside the ``keep_groups`` groups of neighbouring
  experts whose two largest choice scores add up highest; the weights are the chosen s, not renormalized)
  (``score`` = "softmax_all": s = soft-max over all logits, the choice likewise by s + correction, the weights are the chosen s
  over their sum; a group may be judged by its one largest choice score, ``group_best`` = 1)
  all weights are multiplied by ``weight_scale``; the last ``identity`` outputs of the router are experts that return their input
  expert(h) = W_down (g sigmoid(alpha g) (u + shift)),  g = min(W_gate h, limit),  u = clamp(W_up h, -limit, limit)
  (limit infinite, alpha 1, shift 0: W_down (silu(W_gate h) * W_up h)); or, without a gate matrix, W_down act(W_up h)
  y = sum over the chosen experts of weight * expert(h)  +  shared(h)
  (the shared expert may be multiplied by sigmoid(w h), one number per token: w is one more row of the router's matrix)

The experts' matrices are stacked at load time ([experts, ff, W] and [experts, W, ff]).  Steps of few rows run one
workgroup per (token, chosen expert), which streams that expert's matrices; steps of many rows sort the (token, expert)
pairs by expert on the device and run the experts as grouped products of 16-row tiles (``csrc/moe.hip``).  Nothing
depends on the host knowing which experts were chosen, so a step can be captured.
"""

from __future__ import annotations

import torch

from ..config.spec import PlainFFSpec
from ..kernels import ops
from . import registry
from .linear import GatedWeights, LinearWeight


class MoE:
    graph_safe = True
    takes_layouts = True

    def __init__(self, spec, prefix: str) -> None:
        outputs = spec.experts + spec.identity  # what the router chooses from
        if not 0 < spec.top <= outputs or spec.top > ops.MOE_MAX_TOP or outputs > ops.MOE_MAX_EXPERTS or spec.experts < 1 or spec.identity < 0:
            raise ValueError(f"{spec.top} of {outputs} experts (at most {ops.MOE_MAX_TOP} of {ops.MOE_MAX_EXPERTS})")
        if spec.score not in ops.MOE_SCORES:
            raise ValueError(f"score={spec.score!r}: use one of {sorted(ops.MOE_SCORES)}")
        if spec.correction_name and spec.score == "softmax":
            raise ValueError("a correction on the choice belongs to scores, not to logits")
        if spec.groups < 1 or outputs % spec.groups or not 1 <= spec.keep_groups <= spec.groups or spec.top > spec.keep_groups * (outputs // spec.groups):
            raise ValueError(f"{outputs} experts in {spec.groups} groups of which {spec.keep_groups} are kept, {spec.top} chosen")
        if spec.group_best not in (1, 2):
            raise ValueError(f"group_best={spec.group_best}: a group is judged by its best or its two best")
        # experts without gate matrices: their activation by name (None: gated experts)
        self.act = spec.expert.activation if isinstance(spec.expert, PlainFFSpec) else None
        if self.act is not None and self.act not in ops.ACTIVATIONS:
            raise ValueError(f"activation {self.act!r} of the experts is not known (known: {sorted(ops.ACTIVATIONS)})")
        if spec.shared is not None and (isinstance(spec.shared, PlainFFSpec) != (self.act is not None)):
            raise ValueError("the shared expert has the form of the others")
        if spec.shared_gate_name and (spec.shared is None or spec.router_bias_name):
            raise ValueError("a gate on the shared expert goes with a shared expert and a router without a bias")
        self.spec, self.prefix = spec, prefix
        self.outputs = outputs

    def _expert(self, e: int, which: int) -> str:
        return f"{self.prefix}{self.spec.expert_prefix}{e}.{self.spec.names[which]}"

    def _shared(self, which: int) -> str:
        return self.prefix + self.spec.shared_prefix + self.spec.names[which]

    def wanted(self) -> dict:
        s = self.spec
        ff = s.expert.intermediate
        out = {self.prefix + s.router_name: ((self.outputs, s.hidden), "linear")}
        if s.router_bias_name:
            out[self.prefix + s.router_bias_name] = ((self.outputs,), "bias")
        if s.correction_name:
            out[self.prefix + s.correction_name] = ((self.outputs,), "bias")
        for e in range(s.experts):
            if self.act is None:
                out[self._expert(e, 0)] = ((ff, s.hidden), "linear")
            out[self._expert(e, 1)] = ((ff, s.hidden), "linear")
            out[self._expert(e, 2)] = ((s.hidden, ff), "linear")
        if s.shared is not None:
            sf = s.shared.intermediate
            if self.act is None:
                out[self._shared(0)] = ((sf, s.hidden), "linear")
            if s.shared_gate_name:
                out[self.prefix + s.shared_prefix + s.shared_gate_name] = ((1, s.hidden), "linear")
            out[self._shared(1)] = ((sf, s.hidden), "linear")
            out[self._shared(2)] = ((s.hidden, sf), "linear")
        return out

    def load(self, get, dtype, device, layouts: str = "both") -> None:
        s = self.spec
        plain = layouts == "both"
        stack = lambda which: torch.stack([get(self._expert(e, which)).to(device=device, dtype=dtype) for e in range(s.experts)]).contiguous()
        self.gate, self.up, self.down = (stack(0) if self.act is None else None), stack(1), stack(2)
        router = [get(self.prefix + s.router_name)]
        if s.shared_gate_name:
            router.append(get(self.prefix + s.shared_prefix + s.shared_gate_name))
        self.router = torch.cat([t.to(device=device, dtype=torch.float32) for t in router]).contiguous()
        self.extra = self.router.shape[0] - self.outputs
        f32 = lambda name: get(self.prefix + name).to(device=device, dtype=torch.float32).contiguous() if name else None
        self.router_bias, self.correction = f32(s.router_bias_name), f32(s.correction_name)
        self.shared_in = self.shared_gated = self.shared_out = None
        if s.shared is not None:
            to = lambda i: get(self._shared(i)).to(device=device, dtype=dtype)
            if self.act is None and (s.shared.limit, s.shared.alpha, s.shared.shift) == (float("inf"), 1.0, 0.0):
                # the gated SiLU form: few rows apply the activation in the streaming product's epilogue
                self.shared_gated = GatedWeights(to(0), to(1), keep_plain=plain)
            else:
                gu = torch.cat([to(i) for i in ((0, 1) if self.act is None else (1,))]).contiguous()
                self.shared_in = LinearWeight(gu, keep_plain=plain)
            self.shared_out = LinearWeight(get(self._shared(2)).to(device=device, dtype=dtype).contiguous(), keep_plain=plain)

    def forward(self, ctx, x, out: torch.Tensor | None = None):
        s = self.spec
        n, take = x.shape[0], ctx.arena.take
        sel, wt = take((n, s.top), torch.int32), take((n, s.top), torch.float32)
        z = take((n, self.outputs + self.extra), torch.float32)
        ops.moe_route(x, self.router, self.router_bias, s.top, sel, wt, logits=z, score=s.score, correction=self.correction,
                      groups=s.groups, keep=s.keep_groups, extra=self.extra, group_best=s.group_best, scale=s.weight_scale)
        base = None
        if s.shared is not None:
            sf = s.shared.intermediate
            if self.shared_gated is not None:
                act = self.shared_gated(ctx, x, out=take((n, sf), x.dtype))
            elif self.act is None:
                gu = self.shared_in(x, out=take((n, 2 * sf), x.dtype), arena=ctx.arena, plain_copy=not ctx.captured)
                act = ops.clipped_glu(gu, s.shared.limit, s.shared.alpha, out=take((n, sf), x.dtype), shift=s.shared.shift)
            else:
                act = self.shared_in(x, out=take((n, sf), x.dtype), arena=ctx.arena, plain_copy=not ctx.captured, act=self.act)
            base = self.shared_out(act, out=take((n, s.hidden), x.dtype), arena=ctx.arena, plain_copy=not ctx.captured)
        e = s.expert
        form = (e.limit, e.alpha, take, e.shift) if self.act is None else (0.0, 0.0, take, 0.0, self.act)
        parts = ops.moe_experts(x, self.gate, self.up, self.down, sel, wt, *form)
        return ops.moe_combine(parts, base, out if out is not None else take((n, s.hidden), x.dtype),
                               gate=z[:, self.outputs] if s.shared_gate_name else None,
                               identity=(sel, wt, x, s.experts) if s.identity else None)


registry.register("ffn", "moe", MoE)
