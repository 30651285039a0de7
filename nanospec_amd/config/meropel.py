"""The Meropel decoder's configuration, read from its own config.json keys.

A Meropel model is a list of layers over a 32-bit residual stream with a norm in front of each sublayer and one behind it,
x <- x + norm1b(mixer(norm1(x))), x <- x + norm2b(ff(norm2(x))); the stream starts from the sum of the token's embedding and a
row of a second table that the token and the one before it choose.  Mixers:
  parallel    left_scale * left + right_scale * right.  left: grouped soft-max attention, a rotation of the first rot.dims channels
              (pairs i and i + dims/2), values of their own size, one sigmoid gate per head.  right: Mamba's selective scan.
  gla         gated linear attention: a decay per token and key channel, sigmoid(.)^(1/tau).
  parallel_2  half the sum of both outputs, each behind an RMS norm over the width.  left: grouped soft-max attention with biases on
              q, k and v, an RMS norm over the whole of q and of k, a rotation (pairs 2i and 2i + 1).  right: Mamba-2.
Feed-forwards: "dense" (gated SiLU) and "moe" (experts of that form; the scores are the soft-max over all of the router's outputs,
a stored correction on the choice, groups judged by their best, identity experts, a scale; optionally a shared expert).  config.json:

    architecture  "Meropel"
    vocab, width
    logit_scale                          on the head's logits                                     (absent: 1)
    norm.eps
    embedding.bigram                     {"buckets", "mul_prev", "mul_cur"}                       (absent: no second table)
    layers[i]                            {"type", "mixer": {...}, "mlp": {...} | null}
      parallel    left {heads, kv_heads, dim, vdim, scale, rot {base, dims}}, right {inner, state, dt_rank, conv}, left_scale,
                  right_scale                                                                     (scales absent: 1)
      gla         heads, dim, vdim, tau
      parallel_2  left as above, right {heads, vdim, state, groups, conv, norm_groups}
      mlp dense   ff
      mlp moe     expert.ff, router {experts, top, scale, identity, groups {count, keep}}, shared {ff} | absent

Tensor names: embed, bigram, head, final.norm, and per layer l<i>.norm1, .norm1b, .norm2, .norm2b, l<i>.mix.* (two mixers: .left.*
and .right.*, parallel_2 also .left.out and .right.out), l<i>.mlp.{gate,up,down}, or l<i>.mlp.e<j>.*, .router, .correction, .shared.*.
The inner size of a gla layer's two decay matrices is that of the stored tensors.
"""

from __future__ import annotations

from dataclasses import dataclass, field

from .registry import register_architecture
from .spec import (AttentionSpec, ClippedGLUSpec, GatedLinearSpec, LayerCall, ModelSpec, MoESpec, NoPositionSpec, PairEmbeddingSpec, ParallelMixerSpec,
                   RMSNormSpec, RopeSpec, SelectiveScanSpec, StateSpaceSpec, StreamBlockSpec, SwiGLUSpec)

MIXERS = ("parallel", "gla", "parallel_2")


@dataclass(frozen=True)
class MeropelFF:
    kind: str  # "dense" | "moe"
    ff: int  # inner size (of one expert for "moe")
    experts: int = 0
    top: int = 0
    scale: float = 1.0
    identity: int = 0
    groups: int = 1
    keep: int = 1
    shared_ff: int = 0  # 0: no shared expert

    @classmethod
    def from_hf(cls, mlp: dict) -> "MeropelFF":
        kind = mlp.get("kind", "dense")
        if kind == "dense":
            return cls(kind=kind, ff=int(mlp["ff"]))
        if kind != "moe":
            raise ValueError(f"unknown feed-forward kind {kind!r}; known: 'dense', 'moe'")
        r, shared = mlp["router"], mlp.get("shared") or {}
        g = r.get("groups") or {}
        count = int(g.get("count", 1))
        return cls(kind=kind, ff=int(mlp["expert"]["ff"]), experts=int(r["experts"]), top=int(r["top"]), scale=float(r.get("scale", 1.0)),
                   identity=int(r.get("identity") or 0), groups=count, keep=int(g.get("keep", count)), shared_ff=int(shared.get("ff", 0)))

    def to_hf(self) -> dict:
        if self.kind == "dense":
            return {"kind": "dense", "ff": self.ff}
        router: dict = {"experts": self.experts, "top": self.top, "scale": self.scale}
        if self.identity:
            router["identity"] = self.identity
        if self.groups > 1:
            router["groups"] = {"count": self.groups, "keep": self.keep}
        out: dict = {"kind": "moe", "expert": {"ff": self.ff}, "router": router}
        if self.shared_ff:
            out["shared"] = {"ff": self.shared_ff}
        return out


@dataclass(frozen=True)
class MeropelAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_dims: int = 0  # rotated channels of a head; 0: no rotation
    rot_base: float = 10000.0

    @classmethod
    def from_hf(cls, m: dict) -> "MeropelAttention":
        rot = m.get("rot") or {}
        heads, dim = int(m["heads"]), int(m["dim"])
        return cls(heads=heads, kv_heads=int(m.get("kv_heads", heads)), dim=dim, vdim=int(m.get("vdim", dim)), scale=float(m["scale"]),
                   rot_dims=int(rot.get("dims", dim)) if rot else 0, rot_base=float(rot.get("base", 10000.0)))

    def to_hf(self) -> dict:
        out: dict = dict(heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim, scale=self.scale)
        if self.rot_dims:
            out["rot"] = {"base": self.rot_base, "dims": self.rot_dims}
        return out


@dataclass(frozen=True)
class MeropelScan:  # the right side of "parallel"
    inner: int
    state: int
    dt_rank: int
    conv: int


@dataclass(frozen=True)
class MeropelStateSpace:  # the right side of "parallel_2"
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int


@dataclass(frozen=True)
class MeropelGLA:
    heads: int
    dim: int
    vdim: int
    tau: float
    decay_rank: int | None = None  # inner size of the decay's two matrices; None: read from the checkpoint


@dataclass(frozen=True)
class MeropelLayer:
    type: str  # one of MIXERS
    left: MeropelAttention | None = None
    right: MeropelScan | MeropelStateSpace | None = None
    left_scale: float = 1.0
    right_scale: float = 1.0
    gla: MeropelGLA | None = None
    mlp: MeropelFF | None = None

    @classmethod
    def from_hf(cls, entry: dict) -> "MeropelLayer":
        kind, m, mlp = entry["type"], entry["mixer"], entry.get("mlp")
        if kind not in MIXERS:
            raise ValueError(f"unknown mixer type {kind!r}; known: {MIXERS}")
        ff = None if mlp is None else MeropelFF.from_hf(mlp)
        if kind == "gla":
            dim = int(m["dim"])
            return cls(type=kind, gla=MeropelGLA(int(m["heads"]), dim, int(m.get("vdim", dim)), float(m["tau"])), mlp=ff)
        left, r = MeropelAttention.from_hf(m["left"]), m["right"]
        if kind == "parallel":
            right = MeropelScan(*(int(r[k]) for k in ("inner", "state", "dt_rank", "conv")))
            return cls(type=kind, left=left, right=right, left_scale=float(m.get("left_scale", 1.0)), right_scale=float(m.get("right_scale", 1.0)), mlp=ff)
        right = MeropelStateSpace(*(int(r[k]) for k in ("heads", "vdim", "state")), groups=int(r.get("groups", 1)), conv=int(r["conv"]),
                                  norm_groups=int(r.get("norm_groups", 1)))
        return cls(type=kind, left=left, right=right, mlp=ff)

    def to_hf(self) -> dict:
        if self.type == "gla":
            g = self.gla
            m: dict = dict(heads=g.heads, dim=g.dim, vdim=g.vdim, tau=g.tau)
        else:
            m = {"left": self.left.to_hf(), "right": dict(self.right.__dict__)}
            if self.type == "parallel":
                m.update(left_scale=self.left_scale, right_scale=self.right_scale)
        return {"type": self.type, "mixer": m, "mlp": None if self.mlp is None else self.mlp.to_hf()}


@dataclass(frozen=True)
class MeropelConfig:
    vocab: int
    width: int
    layers: tuple[MeropelLayer, ...]
    norm_eps: float = 1e-6
    logit_scale: float = 1.0
    bigram: tuple[int, int, int] | None = None  # (buckets, mul_prev, mul_cur)
    eos_token_ids: tuple[int, ...] = field(default_factory=tuple)

    architecture = "Meropel"

    @classmethod
    def from_hf(cls, cfg: dict, generation_cfg: dict | None = None) -> "MeropelConfig":
        if cfg.get("architecture") != cls.architecture and cls.architecture not in (cfg.get("architectures") or []):
            raise ValueError(f"not a {cls.architecture} configuration")
        eos = (generation_cfg or {}).get("eos_token_id", cfg.get("eos_token_id"))
        eos_ids = () if eos is None else tuple(int(e) for e in (eos if isinstance(eos, (list, tuple)) else [eos]))
        b = (cfg.get("embedding") or {}).get("bigram")
        out = cls(
            vocab=int(cfg["vocab"]),
            width=int(cfg["width"]),
            layers=tuple(MeropelLayer.from_hf(e) for e in cfg["layers"]),
            norm_eps=float(cfg["norm"]["eps"]),
            logit_scale=float(cfg.get("logit_scale", 1.0)),
            bigram=None if not b else (int(b["buckets"]), int(b["mul_prev"]), int(b["mul_cur"])),
            eos_token_ids=eos_ids,
        )
        out.validate()
        return out

    def validate(self) -> None:
        if self.vocab <= 0 or self.width <= 0 or not self.layers or (self.bigram is not None and self.bigram[0] <= 0):
            raise ValueError("vocab, width, the number of layers and the pair table's buckets must be positive")
        for i, l in enumerate(self.layers):
            a, r, g, f = l.left, l.right, l.gla, l.mlp
            if a is not None and (min(a.heads, a.kv_heads, a.dim, a.vdim) <= 0 or a.heads % a.kv_heads):
                raise ValueError(f"layer {i}: {a.heads} heads of sizes {a.dim} and {a.vdim} over {a.kv_heads} key/value heads")
            if a is not None and (a.rot_dims % 2 or not 0 <= a.rot_dims <= a.dim):
                raise ValueError(f"layer {i}: rot.dims={a.rot_dims} must be even and at most dim={a.dim}")
            if r is not None and min(r.__dict__.values()) <= 0:
                raise ValueError(f"layer {i}: the sizes of the right mixer must be positive ({r})")
            if isinstance(r, MeropelStateSpace) and (r.heads % r.groups or (r.heads * r.vdim) % r.norm_groups):
                raise ValueError(f"layer {i}: {r.heads} heads of {r.vdim} in {r.groups} groups, normed in {r.norm_groups} parts")
            if g is not None and (min(g.heads, g.dim, g.vdim) <= 0 or not g.tau > 0):
                raise ValueError(f"layer {i}: gla of {g.heads} heads of {g.dim} x {g.vdim}, tau {g.tau}")
            if f is not None and f.ff <= 0:
                raise ValueError(f"layer {i}: inner size {f.ff}")
            if f is not None and f.kind == "moe":
                outputs = f.experts + f.identity
                if f.experts <= 0 or f.identity < 0 or f.groups < 1 or outputs % f.groups or not 0 < f.keep <= f.groups:
                    raise ValueError(f"layer {i}: {f.experts} experts and {f.identity} identity experts in {f.groups} groups of which {f.keep} are kept")
                if not 0 < f.top <= f.keep * (outputs // f.groups):
                    raise ValueError(f"layer {i}: {f.top} experts cannot be chosen from {f.keep} groups of {outputs // f.groups}")

    def to_hf(self) -> dict:
        out = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "logit_scale": self.logit_scale,
               "layers": [l.to_hf() for l in self.layers], "norm": {"eps": self.norm_eps}}
        if self.bigram is not None:
            out["embedding"] = {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), self.bigram))}
        if self.eos_token_ids:
            out["eos_token_id"] = list(self.eos_token_ids)
        return out

    def _attention(self, a: MeropelAttention, interleaved: bool, **options) -> AttentionSpec:
        position = RopeSpec(rotary_dim=a.rot_dims, theta=a.rot_base, interleaved=interleaved) if a.rot_dims else NoPositionSpec()
        return AttentionSpec(hidden=self.width, heads=a.heads, kv_heads=a.kv_heads, head_dim=a.dim, value_dim=a.vdim, position=position,
                             softmax_scale=a.scale, names=("q", "k", "v", "o"), **options)

    def _mixer(self, l: MeropelLayer):
        W, eps = self.width, self.norm_eps
        if l.type == "gla":
            g = l.gla
            return GatedLinearSpec(hidden=W, heads=g.heads, key_dim=g.dim, value_dim=g.vdim, tau=g.tau, query_scale=g.dim**-0.5, norm_eps=eps,
                                   decay_rank=g.decay_rank)
        r = l.right
        if l.type == "parallel":
            return ParallelMixerSpec(left=self._attention(l.left, False, head_gate=True),
                                     right=SelectiveScanSpec(hidden=W, inner=r.inner, state=r.state, dt_rank=r.dt_rank, conv=r.conv),
                                     left_scale=l.left_scale, right_scale=l.right_scale)
        return ParallelMixerSpec(left=self._attention(l.left, True, bias=True, out_bias=False, whole_norm_eps=eps),
                                 right=StateSpaceSpec(hidden=W, heads=r.heads, value_dim=r.vdim, state=r.state, groups=r.groups, conv=r.conv,
                                                      norm_groups=r.norm_groups, norm_eps=eps),
                                 left_scale=0.5, right_scale=0.5, out_norm_eps=eps)

    def _ffn(self, f: MeropelFF | None):
        if f is None:
            return None
        if f.kind == "dense":
            return SwiGLUSpec(hidden=self.width, intermediate=f.ff, names=("gate", "up", "down"))
        silu = lambda ff: ClippedGLUSpec(intermediate=ff, limit=float("inf"), alpha=1.0, shift=0.0)  # silu(gate) * up
        return MoESpec(hidden=self.width, experts=f.experts, top=f.top, expert=silu(f.ff), shared=silu(f.shared_ff) if f.shared_ff else None,
                       router_bias_name="", score="softmax_all", correction_name="correction", groups=f.groups, keep_groups=f.keep, group_best=1,
                       weight_scale=f.scale, identity=f.identity)

    def model_spec(self) -> ModelSpec:
        norm = RMSNormSpec(dim=self.width, eps=self.norm_eps)
        blocks = []
        for i, l in enumerate(self.layers):
            ffn = self._ffn(l.mlp)
            behind = None if ffn is None else norm
            blocks.append(StreamBlockSpec(prefix=f"l{i}.", mixer_norm=norm, mixer=self._mixer(l), ffn_norm=behind, ffn=ffn, mixer_post_norm=norm,
                                          ffn_post_norm=behind))
        return ModelSpec(
            vocab_size=self.vocab,
            hidden=self.width,
            embed_name="embed",
            layers=tuple(blocks),
            run_order=tuple(LayerCall(i) for i in range(len(self.layers))),
            final_norm=norm,
            final_norm_name="final.norm",
            head_name="head",
            tie_head=False,
            eos_token_ids=self.eos_token_ids,
            logit_scale=self.logit_scale,
            streams=1,
            # what a checkpoint may hold although nothing reads it: the second sublayer's tensors of a layer without a feed-forward
            unread_prefixes=tuple(f"l{i}.{name}" for i, l in enumerate(self.layers) if l.mlp is None for name in ("norm2", "mlp.")),
            pair_embedding=None if self.bigram is None else PairEmbeddingSpec("bigram", *self.bigram),
        )


def _build(cfg: dict, generation_cfg: dict | None):
    config = MeropelConfig.from_hf(cfg, generation_cfg)
    return config, config.model_spec()


register_architecture("Meropel", _build)
