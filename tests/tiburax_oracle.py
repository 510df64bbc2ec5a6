"""A plain float64 implementation of the Tiburax design, one function per mechanism, whole sequences at a time.

It shares nothing with the product path: no packed batches, no cache, no slots, no kernels; every softmax is written
out per query over an explicit list of visible keys, the recurrence walks token by token over an explicit state, every
token runs its own experts.  ``forward(cfg, W, tokens)`` returns the logits of every position and the residual stream
after every layer.  ``W`` maps checkpoint names to tensors, ``cfg`` is the dict of ``config.json``.

The module-level switches plant a mistake, for tests that show that such a mistake is seen.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64
WINDOW_SHIFT = 0         # +-1: the window is one position longer or shorter
KEEP_SHIFT = 0           # +-1: one more or one less of the first tokens stays visible
NO_KEEP = False          # True: no first token is kept
KEPT_AT_EDGE = False     # True: kept tokens are rotated as if they stood just before the window
KV_SHIFT = 0             # 1: query heads read the next key/value head
NORM_FIRST = False       # True: q and k are normed before the rotation instead of after it
MIX_LAST = False         # True: values mix with those of the mixing layer just before, not with the first one's
BIAS_CHOOSES_ONLY = False    # True: the router's bias moves the choice and not the weights
NORM_OF_SUM = False      # True: the norm takes in the residual (a post-norm of the sum)


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def offset_norm(x, w, eps):
    """RMS norm whose weight is stored as an offset from one."""
    return unit_rms(x, eps) * (1.0 + w)


def silu(z):
    return z * torch.sigmoid(z)


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


def frequencies(rot: dict):
    """Turn rates per pair and the magnitude of sine and cosine, with interpolation by parts when ``scaling`` is given."""
    dims, base, sc = int(rot["dims"]), float(rot["base"]), rot.get("scaling")
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not sc:
        return f, 1.0

    def index_of(turns):      # the (fractional) pair that turns this often over the original length
        return dims * math.log(sc["original"] / (turns * 2 * math.pi)) / (2 * math.log(base))
    first = max(math.floor(index_of(sc["fast"])), 0)
    last = min(math.ceil(index_of(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        share = min(max((i - first) / max(last - first, 1e-3), 0.0), 1.0)
        out.append(share * fi / sc["factor"] + (1 - share) * fi)
    return out, 1.0 + 0.1 * math.log(sc["factor"])


def rotate_halves(x, pos: float, rot: dict):
    """x [..., d]: entries i and i + dims/2 below ``dims`` turn by pos * f_i; the rest pass."""
    f, mag = frequencies(rot)
    h, y = len(f), x.clone()
    for i in range(h):
        c, s = math.cos(pos * f[i]) * mag, math.sin(pos * f[i]) * mag
        u, v = x[..., i], x[..., i + h]
        y[..., i] = u * c - v * s
        y[..., i + h] = v * c + u * s
    return y


def visible(i: int, mask: dict | None):
    """The key positions that position i sees."""
    if not mask:
        return list(range(i + 1))
    size = int(mask["size"]) + WINDOW_SHIFT
    keep = 0 if NO_KEEP else int(mask.get("keep_first", 0)) + KEEP_SHIFT
    return [j for j in range(i + 1) if i - j < size or j < keep]


def attend(q, keys, values, scale, cap, mask, edge_keys=None):
    """One head: q [n, d], keys [n, d], values [n, dv].  ``edge_keys(i, j)`` replaces key j for query i (a planted
    mistake)."""
    out = torch.zeros(q.shape[0], values.shape[1], dtype=F64)
    for i in range(q.shape[0]):
        js = visible(i, mask)
        k = keys[js] if edge_keys is None else torch.stack([edge_keys(i, j) for j in js])
        s = (k @ q[i]) * scale
        if cap:
            s = cap * torch.tanh(s / cap)
        e = torch.exp(s - s.max())
        out[i] = (e[:, None] * values[js]).sum(0) / e.sum()
    return out


def attention(W, p, m, h, eps, v_other=None):
    """Returns the mixer's output and its values ``[n, G * dv]`` (mixed with ``v_other`` when given)."""
    n = h.shape[0]
    H, dk, dv = (int(m[k]) for k in ("heads", "dim", "vdim"))
    G, rot = int(m.get("kv_heads", H)), m["rot"]
    g = lambda name: W[p + name].to(F64)      # noqa: E731
    q0, k0, v = (h @ g("q").t()).view(n, H, dk), (h @ g("k").t()).view(n, G, dk), h @ g("v").t()
    if v_other is not None:
        lam = g("vmix").reshape(())
        v = (1 - lam) * v + lam * v_other
    if NORM_FIRST:
        turn = lambda x, pos: rotate_halves(unit_rms(x, eps), pos, rot)      # noqa: E731
    else:
        turn = lambda x, pos: unit_rms(rotate_halves(x, pos, rot), eps)      # noqa: E731
    q = torch.stack([turn(q0[t], t) for t in range(n)])
    k = torch.stack([turn(k0[t], t) for t in range(n)])
    vh, out, mask = v.view(n, G, dv), torch.zeros(n, H, dv, dtype=F64), m.get("mask")
    for hd in range(H):
        kv = (hd // (H // G) + KV_SHIFT) % G
        edge = None
        if KEPT_AT_EDGE:
            def edge(i, j, kv=kv):
                lo = i - int(mask["size"]) + 1
                return k[j, kv] if j >= lo else turn(k0[j, kv], lo - int(mask["keep_first"]) + j)
        out[:, hd] = attend(q[:, hd], k[:, kv], vh[:, kv], float(m["scale"]), float(m.get("softcap") or 0.0), mask, edge)
    return out.reshape(n, H * dv) @ g("o").t(), v


def selective_scan(W, p, m, h):
    """Per channel c and state n: S <- exp(-dt e^A_log) S + dt x B, y = S . C + D x, gated by silu(z)."""
    n = h.shape[0]
    inner, N, R = int(m["inner"]), int(m["state"]), int(m["dt_rank"])
    g = lambda name: W[p + name].to(F64)      # noqa: E731
    xz = h @ g("in").t()
    x, z = xz[:, :inner], xz[:, inner:]
    x = silu(causal_conv(x, g("conv")) + g("conv.b"))
    dbc = x @ g("x").t()
    pre = dbc[:, :R] @ g("dt").t() + g("dt.b")
    dt = pre.clamp(min=0) + torch.log1p(torch.exp(-pre.abs()))
    B, C = dbc[:, R:R + N], dbc[:, R + N:]
    A = -torch.exp(g("A_log"))
    S = torch.zeros(inner, N, dtype=F64)
    y = torch.zeros(n, inner, dtype=F64)
    for t in range(n):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + g("D") * x[t]
    return (y * silu(z)) @ g("o").t()


def glu_expert(W, q, u):
    g = lambda name: W[q + name].to(F64)      # noqa: E731
    return g("down") @ (silu(g("gate") @ u) * (g("up") @ u))


def experts(W, p, mlp, h):
    """Every token: the ``top`` largest of the biased logits, weighted by the softmax over those, plus the shared
    expert."""
    top = int(mlp["router"]["top"])
    plain = h @ W[p + "router"].to(F64).t()
    z = plain + W[p + "router.b"].to(F64)
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        ids = torch.topk(z[t], top).indices
        w = torch.softmax((plain if BIAS_CHOOSES_ONLY else z)[t, ids], -1)
        for e, we in zip(ids.tolist(), w):
            y[t] = y[t] + we * glu_expert(W, f"{p}e{e}.", h[t])
        if mlp.get("shared") is not None:
            y[t] = y[t] + glu_expert(W, p + "shared.", h[t])
    return y


def forward(cfg: dict, W: dict, tokens):
    eps = float(cfg["norm"]["eps"])

    def join(x, y, name):
        w = W[name].to(F64)
        return offset_norm(x + y, w, eps) if NORM_OF_SUM else x + offset_norm(y, w, eps)
    x = W["embed"].to(F64)[torch.tensor(list(tokens))] * float(cfg["embedding"]["scale"])
    first, after = None, []
    for i, lc in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lc["mixer"]
        if lc["type"] == "attention":
            y, v = attention(W, p + "mix.", m, x, eps, first if m.get("v_mix") else None)
            if m.get("v_mix") and (first is None or MIX_LAST):
                first = v
        else:
            y = selective_scan(W, p + "mix.", m, x)
        x = join(x, y, p + "norm1")
        if lc.get("mlp") is not None:
            x = join(x, experts(W, p + "mlp.", lc["mlp"], x), p + "norm2")
        after.append(x.clone())
    return offset_norm(x, W["final.norm"].to(F64), eps) @ W["head"].to(F64).t(), after
