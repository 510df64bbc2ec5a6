"""A plain float64 implementation of the Vefunex design, one function per mechanism, whole sequences at a time.

It shares nothing with the product path: no packed batches, no cache, no slots, no kernels; every softmax is written
out per query, both recurrences walk token by token over explicit states, every token runs its own experts.
``forward(cfg, W, tokens)`` returns the logits of every position and the residual stream after every layer (after the
depth average).  ``W`` maps checkpoint names to tensors, ``cfg`` is the dict of ``config.json``.

The module-level switches plant a mistake, for tests that show that such a mistake is seen.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64
USE_SINK = True          # False: the sink is left out of the denominator
TEMP_SHIFT = 1           # 0: the query temperature steps one position late
FAR_LIMIT = 0            # > 0: attention forgets keys this many positions back or more
KV_SHIFT = 0             # 1: query heads read the next key/value head


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def dynamic_tanh(x, alpha, w, b):
    return torch.tanh(alpha * x) * w + b


def causal_conv(u, w):
    """u [n, C], w [C, taps]: sum_j w[:, j] u_(t - taps + 1 + j), nothing before the start."""
    n, taps = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for t in range(n):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] = y[t] + w[:, j] * u[s]
    return y


def depth_average(weights, streams):
    return sum(weights[j] * streams[j] for j in range(len(streams)))


def rotate_neighbours(x, pos: int, dims: int, base: float):
    """x [..., d]: entries 2i and 2i + 1 below ``dims`` turn by pos * base^(-2i / dims); the rest pass."""
    y = x.clone()
    for i in range(dims // 2):
        a = pos * base ** (-2.0 * i / dims)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i] = u * math.cos(a) - v * math.sin(a)
        y[..., 2 * i + 1] = v * math.cos(a) + u * math.sin(a)
    return y


def temperature(p: int, coef: float, every: int):
    return 1.0 + coef * math.log(math.floor((p + TEMP_SHIFT) / every) + 1.0)


def softmax_sum(q, keys, values, scale, cap=0.0, sink=None):
    """One head: q [n, d], keys [n, d], values [n, dv]; query i sees keys 0..i; ``cap`` bounds the scaled scores,
    ``sink`` adds exp(sink) to every denominator."""
    n = q.shape[0]
    out = torch.zeros(n, values.shape[1], dtype=F64)
    for i in range(n):
        lo = max(0, i - FAR_LIMIT + 1) if FAR_LIMIT else 0
        s = (keys[lo:i + 1] @ q[i]) * scale
        if cap:
            s = cap * torch.tanh(s / cap)
        m = s.max() if sink is None else torch.maximum(s.max(), sink)
        e = torch.exp(s - m)
        den = e.sum() + (torch.exp(sink - m) if sink is not None else 0.0)
        out[i] = (e[:, None] * values[lo:i + 1]).sum(0) / den
    return out


def attention(W, p, m, h, eps):
    """Grouped-query attention without rotation: query temperature by position, values of unit root mean square."""
    n = h.shape[0]
    H, G, dk, dv = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    g = lambda name: W[p + name].to(F64)      # noqa: E731
    q = (h @ g("q").t()).view(n, H, dk)
    k = (h @ g("k").t()).view(n, G, dk)
    v = unit_rms((h @ g("v").t()).view(n, G, dv), eps)
    tm = m["q_temp"]
    q = q * torch.tensor([temperature(t, tm["coef"], tm["every"]) for t in range(n)], dtype=F64)[:, None, None]
    out = torch.zeros(n, H, dv, dtype=F64)
    for hd in range(H):
        kv = (hd // (H // G) + KV_SHIFT) % G
        out[:, hd] = softmax_sum(q[:, hd], k[:, kv], v[:, kv], float(m["scale"]))
    return out.reshape(n, H * dv) @ g("o").t()


def capped_attention(W, p, m, h):
    """Grouped-query attention with rotated q and k, bounded scores, a sink per head and an element-wise gate."""
    n = h.shape[0]
    H, G, dk, dv = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    dims, base = int(m["rot"]["dims"]), float(m["rot"]["base"])
    g = lambda name: W[p + name].to(F64)      # noqa: E731
    q = (h @ g("q").t()).view(n, H, dk)
    k = (h @ g("k").t()).view(n, G, dk)
    v = (h @ g("v").t()).view(n, G, dv)
    q = torch.stack([rotate_neighbours(q[t], t, dims, base) for t in range(n)])
    k = torch.stack([rotate_neighbours(k[t], t, dims, base) for t in range(n)])
    out = torch.zeros(n, H, dv, dtype=F64)
    for hd in range(H):
        kv = (hd // (H // G) + KV_SHIFT) % G
        out[:, hd] = softmax_sum(q[:, hd], k[:, kv], v[:, kv], float(m["scale"]), float(m["softcap"]),
                                 g("sink")[hd] if USE_SINK else None)
    o = out.reshape(n, H * dv) * torch.sigmoid(h @ g("g").t())
    return o @ g("o").t()


def selective_scan(W, p, m, h):
    """Per channel c and state n: S <- exp(-dt e^A_log) S + dt x B, y = S . C + D x, gated by silu(z)."""
    n = h.shape[0]
    inner, N, R = int(m["inner"]), int(m["state"]), int(m["dt_rank"])
    g = lambda name: W[p + name].to(F64)      # noqa: E731
    xz = h @ g("in").t()
    x, z = xz[:, :inner], xz[:, inner:]
    x = silu(causal_conv(x, g("conv")) + g("conv.b"))
    dbc = x @ g("x").t()
    dt = torch.log1p(torch.exp(dbc[:, :R] @ g("dt").t() + g("dt.b")))
    B, C = dbc[:, R:R + N], dbc[:, R + N:]
    A = -torch.exp(g("A_log"))
    S = torch.zeros(inner, N, dtype=F64)
    y = torch.zeros(n, inner, dtype=F64)
    for t in range(n):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + g("D") * x[t]
    return (y * silu(z)) @ g("o").t()


def parallel_mixer(W, p, m, h):
    return float(m["left_scale"]) * capped_attention(W, p + "left.", m["left"], h) \
        + float(m["right_scale"]) * selective_scan(W, p + "right.", m["right"], h)


def gated_linear_attention(W, p, m, h, eps):
    """Per head a [dk, dv] matrix whose rows decay by sigmoid(z)^(1 / tau) and take in k v^T."""
    n = h.shape[0]
    H, dk, dv, tau = int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["tau"])
    g = lambda name: W[p + name].to(F64)      # noqa: E731
    q = (h @ g("q").t()).view(n, H, dk) * dk ** -0.5
    k = (h @ g("k").t()).view(n, H, dk)
    v = (h @ g("v").t()).view(n, H, dv)
    a = (torch.sigmoid((h @ g("a1").t()) @ g("a2").t() + g("a2.b")) ** (1.0 / tau)).view(n, H, dk)
    out = torch.zeros(n, H, dv, dtype=F64)
    for hd in range(H):
        S = torch.zeros(dk, dv, dtype=F64)
        for t in range(n):
            S = a[t, hd][:, None] * S + torch.outer(k[t, hd], v[t, hd])
            out[t, hd] = S.t() @ q[t, hd]
    o = (unit_rms(out, eps) * g("norm")).reshape(n, H * dv) * silu(h @ g("g").t())
    return o @ g("o").t()


def experts(W, p, mlp, h):
    """Every token: the ``top`` experts of the largest sigmoid scores, each fed the token times its score."""
    top = int(mlp["router"]["top"])
    s = torch.sigmoid(h @ W[p + "router"].to(F64).t())
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in torch.topk(s[t], top).indices.tolist():
            u = s[t, e] * h[t]
            g = lambda name: W[f"{p}e{e}.{name}"].to(F64)      # noqa: E731
            y[t] = y[t] + g("down") @ (silu(g("gate") @ u) * (g("up") @ u))
    return y


def forward(cfg: dict, W: dict, tokens):
    eps, m = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])

    def norm(x, name):
        return dynamic_tanh(x, W[name + ".alpha"].to(F64), W[name].to(F64), W[name + ".b"].to(F64))

    def entry(x, p, q):
        h = norm(x, f"{p}norm{q}")
        return h + causal_conv(h, W[f"{p}canon{q}"].to(F64))
    x = W["embed"].to(F64)[torch.tensor(list(tokens))]
    streams, after = [x], []
    for i, lc in enumerate(cfg["layers"]):
        p = f"l{i}."
        h, mx = entry(x, p, 1), lc["mixer"]
        if lc["type"] == "attention":
            y = attention(W, p + "mix.", mx, h, eps)
        elif lc["type"] == "parallel":
            y = parallel_mixer(W, p + "mix.", mx, h)
        else:
            y = gated_linear_attention(W, p + "mix.", mx, h, eps)
        x = x + m * y
        if lc.get("mlp") is not None:
            x = x + m * experts(W, p + "mlp.", lc["mlp"], entry(x, p, 2))
        streams.append(x)
        x = depth_average(W[p + "dwa"].to(F64), streams)
        after.append(x.clone())
    cap = float(cfg["logit_softcap"])
    logits = norm(x, "final.norm") @ W["embed"].to(F64).t()
    return cap * torch.tanh(logits / cap), after
