"""Retention: linear attention with one fixed decay per head, no soft-max and no denominator ("retention").

h [tokens, hidden] is the mixer's input; H heads, D key channels, E value channels.  Per head:
  q = W_q h,  k = W_k h   [D];   v = W_v h   [E];   q and k rotated by their position, k then times key_scale
  S_t = decay S_(t-1) + k_t v_t^T;   o_t = S_t^T q_t                      S [D, E] starts at zero
  y = W_o (o / rms(o) * silu(W_g h))                                     rms per head over E, no weight
Options of the spec: q, k and v pass a SiLU first; one rms over all heads with a weight instead of one per head; a sigmoid
as the gate.  (Lightning attention is all three, without a rotation and with key_scale 1.)
S lives in 32-bit in the request's state slot and is carried from step to step.

One product reads h for q, k, v and the gate together (the matrices are stacked at load time); rotation and scaling
(``retention_prep``), the recurrence and the gated norm (``gated_rms``) are 32-bit kernels.  The recurrence takes a
request's tokens of the step one after the other (``decay_scan``: single tokens, short portions, padding rows, which own
the pad slot) or, from ``CHUNKED_FROM`` tokens on, in chunks whose tokens meet the state and each other as 32-bit matrix
products (``decay_chunks``); the two differ by rounding.
"""

from __future__ import annotations

import numpy as np
import torch

from ..kernels import ops
from . import registry
from .linear import LinearWeight
from .needs import StateNeed

CHUNKED_FROM = 192  # a request that brings at least this many tokens runs in chunks: three kernels that take 40 us however short
#                     the portion is, what the scan's chain takes for about as many tokens (8 heads of 128 x 256: 421 against 79 us
#                     for 2,048 tokens, 109 against 44 for 512, 29 against 40 for 128)


class ChunkPlan:
    """The step's long portions as ``ops.decay_chunks`` walks them (a batch plan, see ``engine.context``): every request that
    brings at least ``CHUNKED_FROM`` tokens cut into chunks.  shape = (chunks, requests left to the scan); a region of a
    fixed shape may hold more chunks than the batch needs: the rest describe nothing."""

    key = "retention.chunks"

    def shape(self, lens) -> tuple[int, int]:
        return sum(-(-n // ops.RETENTION_CHUNK) for n in lens if n >= CHUNKED_FROM), sum(1 for n in lens if n < CHUNKED_FROM)

    def shape_captured(self, rows: int, tokens: int, portions: int) -> tuple[int, int]:
        # every portion may end in a chunk that is not full, and may be too short for chunks
        return (-(-tokens // ops.RETENTION_CHUNK) + portions if tokens >= CHUNKED_FROM else 0), rows + portions

    def ints(self, shape) -> int:
        return ops.RETENTION_CHUNK_INTS * shape[0]

    def fill(self, out: np.ndarray, shape, facts) -> None:
        rows = []
        for b in range(facts.covered):
            n = int(facts.lens[b])
            if n >= CHUNKED_FROM:
                count = -(-n // ops.RETENTION_CHUNK)
                rows += [(b, int(facts.indptr[b]) + i * ops.RETENTION_CHUNK, min(ops.RETENTION_CHUNK, n - i * ops.RETENTION_CHUNK), count if i == 0 else 0)
                         for i in range(count)]
        rows += [(0, 0, 0, 0)] * (shape[0] - len(rows))
        out[: ops.RETENTION_CHUNK_INTS * shape[0]] = np.asarray(rows, dtype=np.int32).reshape(-1)

    @staticmethod
    def view(ctx):
        """-> (chunks as int32 [n, RETENTION_CHUNK_INTS] on the device, requests left to the scan); (None, 1) in a step that has
        no such plan."""
        region, (n, rest) = getattr(ctx, "plans", {}).get(ChunkPlan.key, (None, (0, 1)))
        return (region[: ops.RETENTION_CHUNK_INTS * n].view(n, ops.RETENTION_CHUNK_INTS) if n else None), rest


CHUNKS = ChunkPlan()


def decayed_recurrence(ctx, rows: "ops.DecayRows", state: torch.Tensor, out: torch.Tensor) -> torch.Tensor:
    """A step's decayed recurrence over the state in the requests' slots: long portions in chunks where the sizes allow it, all
    other requests by the scan."""
    takes = ops.decay_chunks_take(rows.key_dim, rows.rows.shape[1], rows.offsets)
    chunks, rest = ChunkPlan.view(ctx) if takes else (None, 1)
    # (the scan first: where decays are per token the chunked form leaves sums in their place, in its own rows)
    if rest:
        ops.decay_scan(rows, state, ctx.qo_indptr, ctx.state_slots, out, skip_from=CHUNKED_FROM if chunks is not None else 0)
    if chunks is not None:
        ops.decay_chunks(rows, state, chunks, ctx.state_slots, ctx.arena.take((chunks.shape[0] * rows.words,), torch.float32), out)
    return out


class Retention:
    graph_safe = True
    takes_layouts = True

    def __init__(self, spec, prefix: str) -> None:
        if spec.heads <= 0 or spec.key_dim <= 0 or spec.value_dim <= 0 or len(spec.decay) != spec.heads:
            raise ValueError(f"retention of {spec.heads} heads of {spec.key_dim} x {spec.value_dim} with {len(spec.decay)} decays")
        if spec.key_dim > ops.RETENTION_MAX_KEY_DIM:
            raise ValueError(f"the recurrence takes key sizes up to {ops.RETENTION_MAX_KEY_DIM}")
        self.spec, self.prefix = spec, prefix
        self.position = registry.build("position", spec.position, prefix)
        if self.position.rotary_dim > spec.key_dim:
            raise ValueError("the rotary part of a head cannot be wider than the head")
        s = spec
        self.qk, self.vw = s.heads * s.key_dim, s.heads * s.value_dim
        # columns of the first product: q | k | v | gate
        self.k_at, self.v_at, self.g_at = self.qk, 2 * self.qk, 2 * self.qk + self.vw
        self.w_in: LinearWeight | None = None
        self.w_out: LinearWeight | None = None
        self.norm: torch.Tensor | None = None

    def _name(self, i: int) -> str:
        return self.prefix + self.spec.names[i]

    def wanted(self) -> dict:
        s = self.spec
        out = {
            self._name(0): ((self.qk, s.hidden), "linear"), self._name(1): ((self.qk, s.hidden), "linear"),
            self._name(2): ((self.vw, s.hidden), "linear"), self._name(3): ((self.vw, s.hidden), "linear"),
            self._name(4): ((s.hidden, self.vw), "linear"), **self.position.wanted(),
        }
        if s.whole_norm_name:
            out[self.prefix + s.whole_norm_name] = ((self.vw,), "norm")
        return out

    def load(self, get, dtype, device, layouts: str = "both") -> None:
        s = self.spec
        plain = layouts == "both"
        rows = -(-(self.g_at + self.vw) // 16) * 16
        w_in = torch.zeros((rows, s.hidden), dtype=dtype, device=device)
        for at, i in ((0, 0), (self.k_at, 1), (self.v_at, 2), (self.g_at, 3)):
            t = get(self._name(i))
            w_in[at : at + t.shape[0]].copy_(t)
        self.w_in = LinearWeight(w_in, keep_plain=plain)
        self.w_out = LinearWeight(get(self._name(4)).to(device=device, dtype=dtype).contiguous(), keep_plain=plain)
        self.decay = torch.tensor([float(d) for d in s.decay], dtype=torch.float32, device=device)
        if s.whole_norm_name:
            self.norm = get(self.prefix + s.whole_norm_name).to(device=device, dtype=torch.float32).contiguous()
        self.position.load(get, dtype, device)
        self._form = dict(interleaved=bool(getattr(self.position, "interleaved", False)), factor=float(getattr(self.position, "factor", 1.0)))

    def cache_need(self):
        s = self.spec
        return StateNeed((s.heads * s.key_dim * s.value_dim,), torch.float32)

    def batch_plans(self) -> list:
        s = self.spec
        return [CHUNKS] if ops.retention_chunks_take(s.heads, s.key_dim, s.value_dim) else []

    def max_positions(self) -> int | None:
        return self.position.max_positions

    def forward(self, ctx, x, cache, owns_cache: bool = True, out: torch.Tensor | None = None):
        s, pos = self.spec, self.position
        n, take = x.shape[0], ctx.arena.take
        if pos.max_positions is not None and ctx.max_position >= pos.max_positions:
            raise ValueError(f"position {ctx.max_position} is beyond the model's {pos.max_positions} positions")
        proj = self.w_in(x, out=take((n, self.w_in.n), x.dtype), arena=ctx.arena, plain_copy=not ctx.captured)
        qkv = ops.retention_prep(proj, (0, self.k_at, self.v_at), ctx.positions, pos.inv_freq, s.heads, s.key_dim, s.value_dim, pos.rotary_dim,
                                 s.key_scale, out=take((n, 2 * self.qk + self.vw), torch.float32), silu=s.qkv_silu, **self._form)
        rows = ops.retention_rows(qkv, self.decay, s.heads, s.key_dim, s.value_dim)
        o = decayed_recurrence(ctx, rows, cache.state, take((n, self.vw), torch.float32))
        gated = ops.gated_rms(o, proj[:, self.g_at : self.g_at + self.vw], self.norm, s.norm_eps, 1 if s.whole_norm_name else s.heads,
                              out=take((n, self.vw), x.dtype), silu=s.gate_silu)
        return self.w_out(gated, out=out if out is not None else take((n, s.hidden), x.dtype), arena=ctx.arena, plain_copy=not ctx.captured)


registry.register("mixer", "retention", Retention)
