"""The selective scan of Mamba ("selective_scan").

h [tokens, hidden] is the mixer's input; c channels (inner), N states a channel, R the rank of the step sizes, K taps.
  [x | z] = W_in h;   x = silu(conv(x) + b)                                short causal convolution per channel
  [r: R | B: N | C: N] = W_x x;   dt = softplus(W_dt r + b_dt)   [c];   A = -exp(A_log)   [c, N]
  S <- S * exp(dt[:, None] A) + (dt x) B^T;   y = S C + D * x             token by token, S [c, N] from zero
  y = W_o (y * silu(z))
Three products (h, x, r), the convolution with its carried inputs (``conv_silu_carry``) and one kernel from the step sizes to
the gated read-out (``selective_scan``; long portions of few states in chunks, ``selective_chunks``); what is not a product is 32-bit.  What a request carries from step to step lives
in its state slot: S [c, N] and the last K - 1 inputs of the convolution [K - 1, c].
"""

from __future__ import annotations

import torch

from ..kernels import ops
from . import registry, retention
from .linear import LinearWeight
from .needs import StateNeed
from .retention import CHUNKS, ChunkPlan


def a_log_law(shape, gen):
    """Logarithms of decay rates 1, 2, .. along the states, a little apart from channel to channel."""
    base = torch.log(torch.arange(1, shape[-1] + 1, dtype=torch.float32, device=gen.device)).expand(shape)
    return base + 0.1 * torch.randn(shape, generator=gen, dtype=torch.float32, device=gen.device)


def step_bias_law(shape, gen):
    """Step sizes of about 0.01 to 0.3 where the token chooses nothing."""
    return torch.empty(shape, dtype=torch.float32, device=gen.device).uniform_(-4.6, -1.2, generator=gen)


def conv_law(shape, gen):
    return torch.empty(shape, dtype=torch.float32, device=gen.device).normal_(0.0, 0.5, generator=gen)


class SelectiveScan:
    graph_safe = True
    takes_layouts = True

    def __init__(self, spec, prefix: str) -> None:
        if spec.inner <= 0 or spec.dt_rank <= 0 or not 1 <= spec.conv <= ops.MAX_CONV_TAPS or not 1 <= spec.state <= ops.SELECTIVE_SCAN_MAX_STATE:
            raise ValueError(f"a selective scan of {spec.inner} channels of {spec.state} states (1 to {ops.SELECTIVE_SCAN_MAX_STATE}) behind {spec.conv} "
                             f"taps (1 to {ops.MAX_CONV_TAPS}), step sizes of rank {spec.dt_rank}")
        self.spec, self.prefix = spec, prefix
        self.conv_off = -(-spec.inner * spec.state // 4) * 4  # where the carried inputs lie in a slot
        self.slot_floats = -(-(self.conv_off + (spec.conv - 1) * spec.inner) // 4) * 4

    def _name(self, i: int) -> str:
        return self.prefix + self.spec.names[i]

    def wanted(self) -> dict:
        s, b = self.spec, self.spec.bias_suffix
        return {
            self._name(0): ((2 * s.inner, s.hidden), "linear"),
            self._name(1): ((s.inner, s.conv), conv_law), self._name(1) + b: ((s.inner,), "bias"),
            self._name(2): ((s.dt_rank + 2 * s.state, s.inner), "linear"),
            self._name(3): ((s.inner, s.dt_rank), "linear"), self._name(3) + b: ((s.inner,), step_bias_law),
            self._name(4): ((s.inner, s.state), a_log_law), self._name(5): ((s.inner,), "ones"),
            self._name(6): ((s.hidden, s.inner), "linear"),
        }

    def load(self, get, dtype, device, layouts: str = "both") -> None:
        s, b = self.spec, self.spec.bias_suffix
        plain = layouts == "both"
        to = lambda name: get(name).to(device=device, dtype=dtype).contiguous()
        f32 = lambda name: get(name).to(device=device, dtype=torch.float32).contiguous()

        def padded(name):  # rows in multiples of 16, so that a row of the product stays aligned
            t = get(name)
            w = torch.zeros((-(-t.shape[0] // 16) * 16, t.shape[1]), dtype=dtype, device=device)
            w[: t.shape[0]].copy_(t)
            return w

        self.w_in = LinearWeight(padded(self._name(0)), keep_plain=plain)
        self.w_x = LinearWeight(padded(self._name(2)), keep_plain=plain)
        self.w_dt = LinearWeight(to(self._name(3)), keep_plain=True)
        self.w_out = LinearWeight(to(self._name(6)), keep_plain=plain)
        self.taps, self.conv_bias = f32(self._name(1)), f32(self._name(1) + b)
        self.dt_bias, self.skip = f32(self._name(3) + b), f32(self._name(5))
        self.A = -torch.exp(f32(self._name(4)))

    def cache_need(self):
        return StateNeed((self.slot_floats,), torch.float32)

    def batch_plans(self) -> list:
        return [CHUNKS] if self.spec.state <= ops.SELECTIVE_CHUNKS_MAX_STATE else []

    def forward(self, ctx, x, cache, owns_cache: bool = True, out: torch.Tensor | None = None):
        s = self.spec
        n, take = x.shape[0], ctx.arena.take
        product = dict(arena=ctx.arena, plain_copy=not ctx.captured)
        proj = self.w_in(x, out=take((n, self.w_in.n), x.dtype), **product)
        u = take((n, s.inner), torch.float32)
        copy = take((n, s.inner), x.dtype) if x.dtype != torch.float32 else None  # what the product through W_x reads
        ops.conv_silu_carry(proj, self.taps, cache.state, self.conv_off, ctx.token_req, ctx.qo_indptr, ctx.state_slots, out=u, bias=self.conv_bias,
                            copy=copy, single=getattr(ctx, "single_tokens", False))
        dbc = self.w_x(u if copy is None else copy, out=take((n, self.w_x.n), x.dtype), **product)
        zdt = self.w_dt(dbc[:, : s.dt_rank], out=take((n, s.inner), x.dtype), **product)
        y = take((n, s.inner), x.dtype)
        rows = ops.SelectiveRows(u, zdt, dbc, s.dt_rank, s.dt_rank + s.state, proj[:, s.inner : 2 * s.inner], self.dt_bias, self.A, self.skip,
                                 cache.state, y)
        chunks, rest = ChunkPlan.view(ctx) if s.state <= ops.SELECTIVE_CHUNKS_MAX_STATE else (None, 1)
        if rest:
            ops.selective_scan(rows, ctx.qo_indptr, ctx.state_slots, skip_from=retention.CHUNKED_FROM if chunks is not None else 0)
        if chunks is not None:
            ops.selective_chunks(rows, chunks, ctx.state_slots, take)
        return self.w_out(y, out=out if out is not None else take((n, s.hidden), x.dtype), **product)


registry.register("mixer", "selective_scan", SelectiveScan)
