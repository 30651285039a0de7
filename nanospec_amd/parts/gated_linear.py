"""Gated linear attention ("gated_linear"): linear attention whose decay, one per token, head and key channel, the input
chooses.

h [tokens, hidden] is the mixer's input; H heads, D key channels, E value channels.  Per head:
  q = W_q h * query_scale,  k = W_k h   [D];   v = W_v h   [E];   alpha = sigmoid(W_a2 (W_a1 h) + b)^(1 / tau)   [D]
  S <- S * alpha (row by row) + k v^T;   o = q^T S                        token by token, S [D, E] from zero
  y = W_o (o / rms(o) * norm * silu(W_g h))                              rms per head over E, one weight [E] for all heads
The request's state slot keeps S, in 32-bit.

One product reads h for q, k, v, the gate and W_a1 together (the matrices are stacked at load time), a second one takes the
thin result through W_a2.  The logarithms of the decays and 32-bit rows of q, k and v (``retention_prep``), the recurrence and the gated
norm are 32-bit kernels; the recurrence is retention's with another decay (``retention.decayed_recurrence``).  S is linear in k, so
query_scale is put on k, where the kernel that makes 32-bit rows of q, k and v multiplies anyway.
"""

from __future__ import annotations

import torch

from ..kernels import ops
from . import registry
from .linear import LinearWeight
from .needs import StateNeed
from .retention import CHUNKS, decayed_recurrence


def _decay_bias_law(shape, gen):
    """Decays that forget over a few to a few hundred tokens once the root of order tau is taken."""
    return torch.empty(shape, dtype=torch.float32, device=gen.device).uniform_(-2.0, 3.0, generator=gen)


class GatedLinear:
    graph_safe = True
    takes_layouts = True

    def __init__(self, spec, prefix: str) -> None:
        if spec.heads <= 0 or spec.key_dim <= 0 or spec.value_dim <= 0 or not spec.tau > 0:
            raise ValueError(f"gated linear attention of {spec.heads} heads of {spec.key_dim} x {spec.value_dim} with tau {spec.tau}")
        if spec.key_dim > ops.RETENTION_MAX_KEY_DIM:
            raise ValueError(f"the recurrence takes key sizes up to {ops.RETENTION_MAX_KEY_DIM}")
        self.spec, self.prefix = spec, prefix
        s = spec
        self.qk, self.vw = s.heads * s.key_dim, s.heads * s.value_dim
        # columns of the first product: q | k | v | gate | the thin part, which starts at a multiple of 8
        self.k_at, self.v_at, self.g_at = self.qk, 2 * self.qk, 2 * self.qk + self.vw
        self.thin_at = -(-(self.g_at + self.vw) // 8) * 8

    def _name(self, i: int) -> str:
        return self.prefix + self.spec.names[i]

    def wanted(self) -> dict:
        s = self.spec
        return {
            self._name(0): ((self.qk, s.hidden), "linear"), self._name(1): ((self.qk, s.hidden), "linear"),
            self._name(2): ((self.vw, s.hidden), "linear"), self._name(3): ((self.vw, s.hidden), "linear"),
            self._name(4): ((s.hidden, self.vw), "linear"), self._name(5): ((s.value_dim,), "norm"),
            self._name(6): ((s.decay_rank, s.hidden), "linear"), self._name(7): ((self.qk, s.decay_rank), "linear"),
            self._name(7) + s.bias_suffix: ((self.qk,), _decay_bias_law),
        }

    def load(self, get, dtype, device, layouts: str = "both") -> None:
        s = self.spec
        plain = layouts == "both"
        a1, a2 = get(self._name(6)), get(self._name(7))
        self.rank = a1.shape[0]
        if a2.shape[1] != self.rank:
            raise ValueError(f"{self.prefix}: the inner sizes of the decay's two matrices differ ({self.rank} and {a2.shape[1]})")
        rows = -(-(self.thin_at + self.rank) // 16) * 16
        w_in = torch.zeros((rows, s.hidden), dtype=dtype, device=device)
        for at, t in ((0, get(self._name(0))), (self.k_at, get(self._name(1))), (self.v_at, get(self._name(2))), (self.g_at, get(self._name(3))),
                      (self.thin_at, a1)):
            w_in[at : at + t.shape[0]].copy_(t)
        self.w_in = LinearWeight(w_in, keep_plain=plain)
        self.w_thin = LinearWeight(a2.to(device=device, dtype=dtype).contiguous(), keep_plain=True)
        self.w_out = LinearWeight(get(self._name(4)).to(device=device, dtype=dtype).contiguous(), keep_plain=plain)
        f32 = lambda name: get(name).to(device=device, dtype=torch.float32).contiguous()
        self.norm, self.decay_bias = f32(self._name(5)), f32(self._name(7) + s.bias_suffix)

    def cache_need(self):
        # (a slot is a whole number of 16-byte pieces)
        return StateNeed((-(-self.qk * self.spec.value_dim // 4) * 4,), torch.float32)

    def batch_plans(self) -> list:
        s = self.spec
        return [CHUNKS] if ops.retention_chunks_take(s.heads, s.key_dim, s.value_dim) else []

    def forward(self, ctx, x, cache, owns_cache: bool = True, out: torch.Tensor | None = None):
        s = self.spec
        n, take = x.shape[0], ctx.arena.take
        proj = self.w_in(x, out=take((n, self.w_in.n), x.dtype), arena=ctx.arena, plain_copy=not ctx.captured)
        z = self.w_thin(proj[:, self.thin_at : self.thin_at + self.rank], out=take((n, self.qk), x.dtype), arena=ctx.arena)
        log_decay = take((n, self.qk), torch.float32)
        qkv = ops.retention_prep(proj, (0, self.k_at, self.v_at), ctx.positions, None, s.heads, s.key_dim, s.value_dim, 0, s.query_scale,
                                 out=take((n, 2 * self.qk + self.vw), torch.float32), decays=(z, self.decay_bias, s.tau, log_decay))
        rows = ops.DecayRows(qkv, (0, self.qk, 2 * self.qk), s.heads, s.key_dim, s.value_dim, log_decay=log_decay)
        o = decayed_recurrence(ctx, rows, cache.state, take((n, self.vw), torch.float32))
        gated = ops.gated_rms(o, proj[:, self.g_at : self.g_at + self.vw], self.norm, s.norm_eps, s.heads, out=take((n, self.vw), x.dtype), silu=True)
        return self.w_out(gated, out=out if out is not None else take((n, s.hidden), x.dtype), arena=ctx.arena, plain_copy=not ctx.captured)


registry.register("mixer", "gated_linear", GatedLinear)
