"""A plain, slow implementation of the Meropel decoder, one function per mechanism, written from the design's equations.
It shares nothing with the package: it reads a configuration as the dictionary that config.json holds and weights as a
dictionary name -> tensor, and runs a whole sequence at once on the CPU in the precision of the weights it is given.

The design: one residual stream x that starts from two embeddings, the token's and that of the pair (token before, token).
Every sublayer has a norm in front and a norm behind, x <- x + norm1b(mixer(norm1(x))), x <- x + norm2b(ff(norm2(x))).
Mixers: "parallel" (attention with a gate per head beside a selective scan, a weight on each), "gla" (linear attention with a
decay per key channel that the input chooses) and "parallel_2" (attention with biases and norms over the whole of q and k beside
a state-space recurrence with one decay per head, the mean of both outputs behind norms of their own).  Feed-forwards: a
gated SiLU one, or a mixture of such experts and of experts that return their input.
"""

from __future__ import annotations

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def pair_rows(tokens: torch.Tensor, buckets: int, mul_prev: int, mul_cur: int) -> torch.Tensor:
    rows = torch.full_like(tokens, buckets)  # the first token has no token before it
    rows[1:] = (tokens[:-1] * mul_prev + tokens[1:] * mul_cur) % buckets
    return rows


def rotate(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float, interleaved: bool) -> torch.Tensor:
    """x [tokens, heads, >= dims]: pair i is channels (i, i + dims / 2), or (2i, 2i + 1) if ``interleaved``; at position p the
    pair, read as a complex number, is multiplied by exp(i a), a = p base^(-2i / dims)."""
    out = x.clone()
    for i in range(dims // 2):
        a, b = (2 * i, 2 * i + 1) if interleaved else (i, i + dims // 2)
        ang = positions.to(torch.float64) * base ** (-2.0 * i / dims)
        c, s = torch.cos(ang).to(x.dtype)[:, None], torch.sin(ang).to(x.dtype)[:, None]
        u, v = x[..., a], x[..., b]
        out[..., a], out[..., b] = u * c - v * s, v * c + u * s
    return out


def grouped_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float) -> torch.Tensor:
    """q [T, H, D], k [T, G, D], v [T, G, E] -> [T, H, E]: every position sees itself and all before it."""
    T, H, _ = q.shape
    G = k.shape[1]
    seen = torch.ones(T, T, dtype=torch.bool).tril()
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        score = (q[:, h] @ k[:, g].T * scale).masked_fill(~seen, float("-inf"))
        out[:, h] = torch.softmax(score, dim=-1) @ v[:, g]
    return out


def gated_attention(h: torch.Tensor, w: dict, p: str, m: dict) -> torch.Tensor:
    T = h.shape[0]
    H, G, D, E = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    pos, rot = torch.arange(T), m["rot"]
    turn = lambda x: rotate(x, pos, int(rot["dims"]), float(rot["base"]), False)
    q, k, v = turn((h @ w[p + "q"].T).view(T, H, D)), turn((h @ w[p + "k"].T).view(T, G, D)), (h @ w[p + "v"].T).view(T, G, E)
    o = grouped_attention(q, k, v, float(m["scale"])) * torch.sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, H * E) @ w[p + "o"].T


def normed_attention(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, D, E = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    pos, rot = torch.arange(T), m["rot"]
    turn = lambda x: rotate(x, pos, int(rot["dims"]), float(rot["base"]), True)
    proj = lambda name: h @ w[p + name].T + w[p + name + ".b"]
    q = turn((rms(proj("q"), eps) * w[p + "q.norm"]).view(T, H, D))
    k = turn((rms(proj("k"), eps) * w[p + "k.norm"]).view(T, G, D))
    return grouped_attention(q, k, proj("v").view(T, G, E), float(m["scale"])).reshape(T, H * E) @ w[p + "o"].T


def causal_conv(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """Per channel sum_j taps[:, j] x[t - (K - 1) + j] + bias, what lies in front of the first token counts as nothing.  x [T, C], taps [C, K]."""
    K = taps.shape[1]
    out = bias.expand_as(x).clone()
    for j in range(K):
        back = K - 1 - j
        if back < len(x):
            out[back:] += taps[:, j] * x[: len(x) - back]
    return out


def selective_scan(x, dt, A, B, C, D, state=None):
    """x, dt [T, c], A [c, n], B, C [T, n], D [c]: S <- exp(dt A) S + dt x B; y = S C + D x.  ``state`` [c, n] is read and updated."""
    S = torch.zeros_like(A) if state is None else state
    y = torch.zeros_like(x)
    for t in range(len(x)):
        S.mul_(torch.exp(dt[t][:, None] * A)).add_((dt[t] * x[t])[:, None] * B[t][None, :])
        y[t] = S @ C[t] + D * x[t]
    return y


def mamba(h: torch.Tensor, w: dict, p: str, m: dict, state=None) -> torch.Tensor:
    inner, N, R = int(m["inner"]), int(m["state"]), int(m["dt_rank"])
    xz = h @ w[p + "in"].T
    x = silu(causal_conv(xz[:, :inner], w[p + "conv"], w[p + "conv.b"]))
    dbc = x @ w[p + "x"].T
    dt = softplus(dbc[:, :R] @ w[p + "dt"].T + w[p + "dt.b"])
    y = selective_scan(x, dt, -torch.exp(w[p + "A_log"]), dbc[:, R : R + N], dbc[:, R + N :], w[p + "D"], state)
    return (y * silu(xz[:, inner:])) @ w[p + "o"].T


def head_decay_scan(x, dt, a, B, C, D, state=None):
    """x [T, H, E], dt [T, H], a, D [H], B, C [T, H, N]: S <- exp(-a dt) S + dt B x^T; y = S^T C + D x, S [H, N, E]."""
    T, H, E = x.shape
    S = torch.zeros(H, B.shape[2], E, dtype=x.dtype) if state is None else state
    y = torch.zeros_like(x)
    for t in range(T):
        S.mul_(torch.exp(-a * dt[t])[:, None, None]).add_((dt[t][:, None] * B[t])[:, :, None] * x[t][:, None, :])
        y[t] = (S * C[t][:, :, None]).sum(1) + D[:, None] * x[t]
    return y


def mamba2(h: torch.Tensor, w: dict, p: str, m: dict, eps: float, state=None) -> torch.Tensor:
    T = h.shape[0]
    H, E, N, G, parts = int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"]), int(m["norm_groups"])
    inner = H * E
    zxbcdt = h @ w[p + "in"].T
    z, xbc, dt = zxbcdt[:, :inner], zxbcdt[:, inner : 2 * inner + 2 * G * N], zxbcdt[:, 2 * inner + 2 * G * N :]
    xbc = silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x = xbc[:, :inner].view(T, H, E)
    spread = lambda t: t.reshape(T, G, N).repeat_interleave(H // G, dim=1)
    B, C = spread(xbc[:, inner : inner + G * N]), spread(xbc[:, inner + G * N :])
    y = head_decay_scan(x, softplus(dt + w[p + "dt_bias"]), torch.exp(w[p + "A_log"]), B, C, w[p + "D"], state)
    y = y.reshape(T, inner) * silu(z)
    y = rms(y.view(T, parts, inner // parts), eps).reshape(T, inner) * w[p + "norm"]
    return y @ w[p + "o"].T


def channel_decay_memory(q, k, v, alpha, state=None):
    """q, k, alpha [T, H, D], v [T, H, E]: S <- diag(alpha) S + k v^T; o = S^T q, S [H, D, E]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype) if state is None else state
    o = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        S.mul_(alpha[t][:, :, None]).add_(k[t][:, :, None] * v[t][:, None, :])
        o[t] = (S * q[t][:, :, None]).sum(1)
    return o


def gla(h: torch.Tensor, w: dict, p: str, m: dict, eps: float, state=None) -> torch.Tensor:
    T = h.shape[0]
    H, D, E = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = (h @ w[p + "q"].T).view(T, H, D) * D**-0.5, (h @ w[p + "k"].T).view(T, H, D), (h @ w[p + "v"].T).view(T, H, E)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    alpha = torch.exp(-softplus(-z) / float(m["tau"])).view(T, H, D)  # sigmoid(z)^(1/tau)
    o = rms(channel_decay_memory(q, k, v, alpha, state), eps) * w[p + "norm"]
    return (o.reshape(T, H * E) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    return float(m["left_scale"]) * gated_attention(h, w, p + "left.", m["left"]) + float(m["right_scale"]) * mamba(h, w, p + "right.", m["right"])


def mean_of_normed(a: torch.Tensor, b: torch.Tensor, wa: torch.Tensor, wb: torch.Tensor, eps: float) -> torch.Tensor:
    return 0.5 * (rms(a, eps) * wa + rms(b, eps) * wb)


def parallel_2(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    return mean_of_normed(normed_attention(h, w, p + "left.", m["left"], eps), mamba2(h, w, p + "right.", m["right"], eps),
                          w[p + "left.out"], w[p + "right.out"], eps)


def gated_ff(h: torch.Tensor, w: dict, p: str) -> torch.Tensor:
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def choose(z: torch.Tensor, correction: torch.Tensor, top: int, groups: int, keep: int, scale: float) -> tuple[torch.Tensor, torch.Tensor]:
    """Router logits [T, n] -> (chosen outputs [T, top], their weights)."""
    s = torch.softmax(z, dim=-1)
    by = s + correction
    T, n = z.shape
    best = by.view(T, groups, n // groups).amax(-1)
    kept = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, best.topk(keep, dim=-1).indices, True)
    sel = by.masked_fill(~kept.repeat_interleave(n // groups, dim=1), float("-inf")).topk(top, dim=-1).indices
    wt = s.gather(1, sel)
    return sel, wt / (wt.sum(-1, keepdim=True) + 1e-20) * scale


def route(h: torch.Tensor, w: dict, p: str, r: dict) -> tuple[torch.Tensor, torch.Tensor]:
    z = h.to(torch.float32) @ w[p + "router"].to(torch.float32).T
    g = r.get("groups") or {"count": 1, "keep": 1}
    return choose(z, w[p + "correction"].to(torch.float32), int(r["top"]), int(g["count"]), int(g["keep"]), float(r.get("scale", 1.0)))


def moe(h: torch.Tensor, w: dict, p: str, mlp: dict) -> torch.Tensor:
    r = mlp["router"]
    sel, wt = route(h, w, p, r)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(sel[t].tolist(), wt[t].tolist()):
            out[t] += a * (gated_ff(h[t : t + 1], w, f"{p}e{e}.")[0] if e < int(r["experts"]) else h[t])
    return out + gated_ff(h, w, p + "shared.") if mlp.get("shared") else out


def mixer(kind: str, h, w, p, m, eps):
    return {"parallel": parallel, "gla": gla, "parallel_2": parallel_2}[kind](h, w, p, m, eps)


def forward(cfg: dict, w: dict, tokens, probe=None) -> torch.Tensor:
    """Logits [tokens, vocab] of one sequence.  ``probe(i, x)`` is called with the stream after every layer."""
    eps = float(cfg["norm"]["eps"])
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    b = (cfg.get("embedding") or {}).get("bigram")
    x = w["embed"][tokens]
    if b:
        x = x + w["bigram"][pair_rows(tokens, int(b["buckets"]), int(b["mul_prev"]), int(b["mul_cur"]))]
    for i, layer in enumerate(cfg["layers"]):
        p, norm = f"l{i}.", lambda y, name: rms(y, eps) * w[f"l{i}.{name}"]
        x = x + norm(mixer(layer["type"], norm(x, "norm1"), w, p + "mix.", layer["mixer"], eps), "norm1b")
        mlp = layer.get("mlp")
        if mlp:
            h = norm(x, "norm2")
            x = x + norm(moe(h, w, p + "mlp.", mlp) if mlp["kind"] == "moe" else gated_ff(h, w, p + "mlp."), "norm2b")
        if probe is not None:
            probe(i, x)
    return ((rms(x, eps) * w["final.norm"]) @ w["head"].T) * float(cfg.get("logit_scale", 1.0))
