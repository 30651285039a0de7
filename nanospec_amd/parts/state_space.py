"""The state-space recurrence of Mamba-2, one decay per token and head ("state_space").

h [tokens, hidden] is the mixer's input; H heads of E channels (inner = H E), N states, G groups, K taps.
  [z | x | B | C | dt] = W_in h, of inner, inner, G N, G N and H;   [x | B | C] = silu(conv([x | B | C]) + b)
  dt = softplus(dt + dt_bias)   [H];   log a = -exp(A_log) dt
  S <- a S + B (dt x)^T;   y = C^T S + D x                                 per head, B and C of its group; S [N, E] from zero
  y = W_o (rms(y * silu(z)) * norm)                                       rms in norm_groups equal parts of the inner channels
One product reads h for everything.  The convolution with its carried inputs (``conv_silu_carry``) leaves 32-bit rows [x | B | C],
in which the recurrence finds its keys (B), queries (C) and values (x): it is retention's with one decay per token and head
(``retention.decayed_recurrence``), the step sizes as weights of k v^T and D as a skip.  What a request carries from step to
step lives in its state slot: S [H, E, N] and the last K - 1 inputs of the convolution [K - 1, inner + 2 G N].
"""

from __future__ import annotations

import torch

from ..kernels import ops
from . import registry
from .linear import LinearWeight
from .mamba import conv_law, step_bias_law
from .needs import StateNeed
from .retention import CHUNKS, decayed_recurrence


def _a_log_law(shape, gen):
    """Logarithms of decay rates of 1 to 16 per unit step."""
    return torch.log(torch.empty(shape, dtype=torch.float32, device=gen.device).uniform_(1.0, 16.0, generator=gen))


class StateSpace:
    graph_safe = True
    takes_layouts = True

    def __init__(self, spec, prefix: str) -> None:
        s = spec
        if s.heads <= 0 or s.value_dim <= 0 or s.groups <= 0 or s.heads % s.groups or not 1 <= s.state <= ops.RETENTION_MAX_KEY_DIM:
            raise ValueError(f"a state-space recurrence of {s.heads} heads of {s.value_dim} in {s.groups} groups with {s.state} states "
                             f"(1 to {ops.RETENTION_MAX_KEY_DIM})")
        if not 1 <= s.conv <= ops.MAX_CONV_TAPS or s.norm_groups <= 0 or (s.heads * s.value_dim) % s.norm_groups:
            raise ValueError(f"{s.conv} taps (1 to {ops.MAX_CONV_TAPS}), {s.heads * s.value_dim} channels normed in {s.norm_groups} parts")
        self.spec, self.prefix = spec, prefix
        self.inner, self.shared = s.heads * s.value_dim, s.groups * s.state
        self.channels = self.inner + 2 * self.shared  # what the convolution runs over
        self.dt_at = self.inner + self.channels
        self.offsets = (self.inner + self.shared, self.inner, 0)  # where q (C), k (B) and v (x) lie in its rows
        self.conv_off = -(-s.heads * s.value_dim * s.state // 4) * 4  # where the carried inputs lie in a slot
        self.slot_floats = -(-(self.conv_off + (s.conv - 1) * self.channels) // 4) * 4

    def _name(self, i: int) -> str:
        return self.prefix + self.spec.names[i]

    def wanted(self) -> dict:
        s = self.spec
        return {
            self._name(0): ((self.dt_at + s.heads, s.hidden), "linear"),
            self._name(1): ((self.channels, s.conv), conv_law), self._name(1) + s.bias_suffix: ((self.channels,), "bias"),
            self._name(2): ((s.heads,), step_bias_law), self._name(3): ((s.heads,), _a_log_law), self._name(4): ((s.heads,), "ones"),
            self._name(5): ((self.inner,), "norm"), self._name(6): ((s.hidden, self.inner), "linear"),
        }

    def load(self, get, dtype, device, layouts: str = "both") -> None:
        s = self.spec
        plain = layouts == "both"
        f32 = lambda name: get(name).to(device=device, dtype=torch.float32).contiguous()
        t = get(self._name(0))
        w_in = torch.zeros((-(-t.shape[0] // 16) * 16, s.hidden), dtype=dtype, device=device)
        w_in[: t.shape[0]].copy_(t)
        self.w_in = LinearWeight(w_in, keep_plain=plain)
        self.w_out = LinearWeight(get(self._name(6)).to(device=device, dtype=dtype).contiguous(), keep_plain=plain)
        self.taps, self.conv_bias = f32(self._name(1)), f32(self._name(1) + s.bias_suffix)
        self.dt_bias, self.a_log, self.skip, self.norm = (f32(self._name(i)) for i in (2, 3, 4, 5))

    def cache_need(self):
        return StateNeed((self.slot_floats,), torch.float32)

    def batch_plans(self) -> list:
        return [CHUNKS] if ops.decay_chunks_take(self.spec.state, self.channels, self.offsets) else []

    def forward(self, ctx, x, cache, owns_cache: bool = True, out: torch.Tensor | None = None):
        s = self.spec
        n, take = x.shape[0], ctx.arena.take
        proj = self.w_in(x, out=take((n, self.w_in.n), x.dtype), arena=ctx.arena, plain_copy=not ctx.captured)
        xbc = ops.conv_silu_carry(proj[:, self.inner :], self.taps, cache.state, self.conv_off, ctx.token_req, ctx.qo_indptr, ctx.state_slots,
                                  out=take((n, self.channels), torch.float32), bias=self.conv_bias, single=getattr(ctx, "single_tokens", False))
        dt, log_decay = take((n, s.heads), torch.float32), take((n, s.heads), torch.float32)
        ops.log_decay_heads(proj[:, self.dt_at : self.dt_at + s.heads], self.dt_bias, self.a_log, dt, log_decay)
        rows = ops.DecayRows(xbc, self.offsets, s.heads, s.state, s.value_dim, kv_heads=s.groups, log_decay=log_decay, value_scale=dt, skip=self.skip)
        y = decayed_recurrence(ctx, rows, cache.state, take((n, self.inner), torch.float32))
        gated = ops.gated_rms(y, proj[:, : self.inner], self.norm, s.norm_eps, s.norm_groups, out=take((n, self.inner), x.dtype), silu=True,
                              gate_first=True)
        return self.w_out(gated, out=out if out is not None else take((n, s.hidden), x.dtype), arena=ctx.arena, plain_copy=not ctx.captured)


registry.register("mixer", "state_space", StateSpace)
