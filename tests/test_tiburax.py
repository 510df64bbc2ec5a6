"""Tiburax on the framework (packed batches, slot state, engine step functions, HIP kernels on a GPU) against the plain
float64 implementation of tests/tiburax_oracle.py.  Every test makes its own small configuration and weights; each
runs on the CPU path and, marked ``gpu``, on the HIP kernels."""
import copy
import json
import math

import pytest
import torch

import tiburax_oracle as O
from llm_in_practise_amd.infer.engine import SamplingParams, ServingEngine
from llm_in_practise_amd.infer.trace import TraceRunner
from llm_in_practise_amd.models.tiburax import TiburaxConfig, TiburaxForCausalLM

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F64 = torch.float64
YARN = {"factor": 3.0, "original": 60, "fast": 4.0, "slow": 0.5}


def moe(experts=5, top=2, ff=20, shared=14):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top},
            **({"shared": {"ff": shared}} if shared else {})}


def att(heads=6, kv_heads=3, dim=10, vdim=7, rot=8, base=90.0, scaling=YARN, scale=0.35, cap=4.0, size=9, keep=3, v_mix=True,
        mlp=None):
    """``scaling`` / ``cap`` / ``size`` of None or 0: that part is left out of the configuration."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "v_mix": v_mix,
         "rot": {"base": base, "dims": rot, **({"scaling": scaling} if scaling else {})}}
    if cap:
        m["softcap"] = cap
    if size:
        m["mask"] = {"size": size, "keep_first": keep}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def mamba(inner=26, state=5, dt_rank=3, conv=4, mlp=None):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}, "mlp": mlp}


def config(layers, width=44, vocab=59, eps=1e-4, scale=3.0):
    return {"architecture": "Tiburax", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps},
            "embedding": {"scale": scale}}


def weights(cfg, seed=0):
    """Random float64 tensors under the checkpoint's names (the first mixing layer's unused blend weight included)."""
    g = torch.Generator().manual_seed(seed)
    Wd = cfg["width"]

    def mat(o, i, s=1.0):
        return torch.randn(o, i, generator=g, dtype=F64) * s / math.sqrt(i)

    def vec(n, mean=0.0, s=0.2):
        return mean + s * torch.randn(n, generator=g, dtype=F64)

    def glu(q, F_):
        W.update({q + "gate": mat(F_, Wd, 1.5), q + "up": mat(F_, Wd, 1.5), q + "down": mat(Wd, F_)})
    W = {"embed": mat(cfg["vocab"], Wd, math.sqrt(Wd) / cfg["embedding"]["scale"]), "head": mat(cfg["vocab"], Wd), "final.norm": vec(Wd)}
    for i, lc in enumerate(cfg["layers"]):
        p, m, q = f"l{i}.", lc["mixer"], f"l{i}.mix."
        W[p + "norm1"] = vec(Wd)
        if lc["type"] == "attention":
            H, G, dk, dv = (m[k] for k in ("heads", "kv_heads", "dim", "vdim"))
            W.update({q + "q": mat(H * dk, Wd), q + "k": mat(G * dk, Wd), q + "v": mat(G * dv, Wd), q + "o": mat(Wd, H * dv)})
            if m["v_mix"]:
                W[q + "vmix"] = vec(1, 0.4, 0.2)[0]
        else:
            n, N, R = m["inner"], m["state"], m["dt_rank"]
            W.update({q + "in": mat(2 * n, Wd), q + "conv": 0.5 * torch.randn(n, m["conv"], generator=g, dtype=F64),
                      q + "conv.b": vec(n), q + "x": mat(R + 2 * N, n, 2.0), q + "dt": mat(n, R, 1.5),
                      q + "dt.b": vec(n, -1.0, 1.0), q + "A_log": vec(n * N, -0.5, 1.5).view(n, N), q + "D": vec(n, 1.0),
                      q + "o": mat(Wd, n)})
        mlp = lc.get("mlp")
        if mlp is not None:
            W[p + "norm2"], q = vec(Wd), p + "mlp."
            W[q + "router"], W[q + "router.b"] = mat(mlp["router"]["experts"], Wd, 1.5), vec(mlp["router"]["experts"], 0.0, 1.0)
            for e in range(mlp["router"]["experts"]):
                glu(f"{q}e{e}.", mlp["expert"]["ff"])
            if mlp.get("shared"):
                glu(q + "shared.", mlp["shared"]["ff"])
    return W


BASE = config([att(mlp=moe()), mamba(mlp=moe(7, 1, 12)), att(heads=3, kv_heads=3, size=5, keep=2, mlp=moe(3, 3, 8, 0)), mamba(inner=19, state=3),
               att(heads=6, kv_heads=3, dim=4, rot=4, size=20, keep=7, mlp=moe())])


def build(cfg, device, seed=0, dtype=torch.float32, tweak=None):
    W = weights(cfg, seed)
    if tweak:
        tweak(W)
    if dtype == torch.bfloat16:
        W = {k: v.to(torch.bfloat16).double() for k, v in W.items()}
    return TiburaxForCausalLM(TiburaxConfig.from_dict(cfg), W, dtype, device), W


def tokens(n, vocab, seed, lo=0):
    return torch.randint(lo, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def err(got, want):
    got, want = got.double().cpu(), want.double()
    return (got - want).abs().max().item() / max(want.abs().max().item(), 1e-9)


def close(got, want, tol=2e-4):
    assert got.shape == want.shape
    e = err(got, want)
    assert e < tol, f"relative error {e:.3g}"


def close16(got, want):
    """bf16 products and activations: root mean square difference over all positions and at the worst one."""
    assert got.shape == want.shape
    d, scale = got.double().cpu() - want, want.pow(2).mean().sqrt()
    e, worst = d.pow(2).mean().sqrt() / scale, d.pow(2).mean(-1).sqrt().max() / scale
    assert e < 0.02 and worst < 0.12, f"relative rms error {e:.3g}, at the worst position {worst:.3g}"


def replay(lm, max_tokens, steps):
    """steps: list of (entries, end); every entry asks for all its tokens.  Returns {id: logits [n, vocab]}."""
    r, out = TraceRunner(lm, max_tokens), {}
    for entries, end in steps:
        es = [{"id": i, "tokens": t, "want": list(range(len(t)))} for i, t in entries]
        got = r.step(es, end)
        o = 0
        for i, t in entries:
            out[i] = torch.cat([out[i], got[o:o + len(t)]]) if i in out else got[o:o + len(t)]
            o += len(t)
    return out


def logits_of(cfg, W, toks):
    return O.forward(cfg, W, toks)[0]


def decoding(toks, cut, name="a"):
    return [([(name, toks[:cut])], [])] + [([(name, [t])], []) for t in toks[cut:]]


def portions(toks, cuts, name="a"):
    steps, at = [], 0
    for n in cuts:
        steps.append(([(name, toks[at:at + n])], []))
        at += n
    assert at == len(toks)
    return steps


class planted:
    """One of the oracle's switches set to a mistake for a while."""

    def __init__(self, **kw):
        self.kw = kw

    def __enter__(self):
        self.old = {k: getattr(O, k) for k in self.kw}
        for k, v in self.kw.items():
            setattr(O, k, v)

    def __exit__(self, *a):
        for k, v in self.old.items():
            setattr(O, k, v)


def _check(device, layers, T=23, tweak=None, seed=1, decode_from=None, tol=2e-4, **kw):
    cfg = config(layers, **kw)
    lm, W = build(cfg, device, seed, tweak=tweak)
    toks = tokens(T, cfg["vocab"], seed)
    want = logits_of(cfg, W, toks)
    close(replay(lm, T, [([("a", toks)], ["a"])])["a"], want, tol)
    if decode_from is not None:
        close(replay(lm, T, decoding(toks, decode_from))["a"], want, tol)
    return cfg, W, toks, want


# --------------------------------------------------------------------------------------- each mechanism alone
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kw", [dict(), dict(heads=1, kv_heads=1, dim=2, vdim=3, rot=2, size=1, keep=1), dict(heads=5, kv_heads=5, dim=12, vdim=12, rot=0, size=4, keep=0),
                                dict(heads=8, kv_heads=2, dim=16, vdim=5, rot=16, cap=0, size=7, keep=30), dict(heads=4, kv_heads=1, dim=6, vdim=32, rot=2, size=0),
                                dict(scaling=None, size=40), dict(cap=0.6, scale=2.0, v_mix=False), dict(heads=2, kv_heads=1, dim=36, vdim=8, rot=24, size=6, keep=6)])
def test_attention_alone(device, kw):
    """MHA, GQA and MQA, dim != vdim and equal, rotation of none, some and all entries with and without frequency scaling,
    caps that bind and none, no mask, windows of one token and longer than the sequence, kept tokens that outlast it.
    Query heads that read a wrong key/value head and a norm before the rotation are seen by the oracle."""
    cfg, W, toks, want = _check(device, [att(**kw), att(**kw)], decode_from=9)
    m = cfg["layers"][0]["mixer"]
    if m["kv_heads"] > 1:
        with planted(KV_SHIFT=1):
            assert err(logits_of(cfg, W, toks), want) > 1e-2
    if m["rot"]["dims"] > 2 and "scaling" in m["rot"]:
        with planted(NORM_FIRST=True):
            assert err(logits_of(cfg, W, toks), want) > 1e-3
    if "mask" in m and 1 < m["mask"]["size"] < 20 and m["mask"]["keep_first"] < 20:
        for mistake in (dict(WINDOW_SHIFT=1), dict(WINDOW_SHIFT=-1), dict(KEEP_SHIFT=1)):
            with planted(**mistake):
                assert err(logits_of(cfg, W, toks), want) > 1e-3, mistake


@pytest.mark.parametrize("scaling", [YARN, dict(YARN, factor=1.0), dict(YARN, fast=1e9, slow=1e-9), dict(YARN, fast=0.9, slow=0.8), dict(YARN, original=4, fast=50.0)])
@pytest.mark.parametrize("dims,base", [(2, 10.0), (8, 90.0), (64, 500000.0)])
def test_frequency_table(scaling, dims, base):
    """Ramps inside the table, over all of it, before it and with equal ends."""
    from llm_in_practise_amd.ops.attention import rotary_table
    f, mag = rotary_table(dims, base, scaling)
    want, m = O.frequencies({"dims": dims, "base": base, "scaling": scaling})
    close(f, torch.tensor(want, dtype=F64), 1e-6)
    assert abs(mag - m) < 1e-12


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("half", [True, False])
@pytest.mark.parametrize("H,G,dk,dv,dims", [(4, 2, 8, 12, 8), (4, 2, 10, 7, 6), (3, 3, 24, 4, 16), (8, 2, 64, 64, 64), (2, 1, 128, 20, 40), (2, 2, 200, 8, 200),
                                            (2, 1, 300, 4, 24), (1, 1, 66, 6, 66), (20, 5, 32, 16, 0)])
def test_rotation_norm_and_value_blend_on_a_cache(device, half, H, G, dk, dv, dims):
    """rope_kv_store with the heads' norms and the value blend, alone and beside the query temperature and unit-RMS values:
    every lane layout, with and without 16-byte rows, rotated parts that end inside a head."""
    from llm_in_practise_amd.models.common import SeqBatch, SeqStateCache
    from llm_in_practise_amd.ops.attention import rope_kv_store, rotary_table
    T, eps, lam = 7, 1e-2, 0.3
    u = torch.randn(T, (H + G) * dk + G * dv, generator=torch.Generator().manual_seed(1))
    rot = {"dims": dims, "base": 30.0, "scaling": YARN}
    f, mag = rotary_table(dims, 30.0, YARN if dims else None)
    freq = O.frequencies(rot)[0] if dims else []
    for start, temp, v_eps in ((0, None, None), (37, (0.7, 8), 1e-3)):
        cache = SeqStateCache([{"k": ((G * dk,), "kv"), "v": ((G * dv,), "kv"), "w": ((G * dv,), "kv")}], 3, 64, torch.float32, device)
        sb, st = SeqBatch.packed(cache, [2], [T], [start]), cache.layers[0]
        st["w"].copy_(torch.randn(st["w"].shape, generator=torch.Generator().manual_seed(2)))
        q = rope_kv_store(u.to(device), H * dk, G * dk, H, G, f.to(device), dims, st["k"], st["v"], sb, half, mag, temp=temp, v_eps=v_eps,
                          qk_eps=eps, v_first=None if v_eps else (st["w"], lam))
        for t in range(T):
            p = start + t
            for h in range(H + G):
                x = u[t, h * dk:(h + 1) * dk].double()
                if dims and half:
                    x = O.rotate_halves(x, p, rot)
                elif dims:
                    y = x.clone()
                    for i, fi in enumerate(freq):
                        c, s = mag * math.cos(p * fi), mag * math.sin(p * fi)
                        y[2 * i], y[2 * i + 1] = x[2 * i] * c - x[2 * i + 1] * s, x[2 * i + 1] * c + x[2 * i] * s
                    x = y
                x = O.unit_rms(x, eps)
                if temp and h < H:
                    x = x * (1 + temp[0] * math.log((p + 1) // temp[1] + 1))
                got = q[t, h * dk:(h + 1) * dk] if h < H else st["k"][2, p, (h - H) * dk:(h - H + 1) * dk]
                close(got, x, 2e-5)
            v = u[t, (H + G) * dk:].double()
            v = O.unit_rms(v.view(G, dv), v_eps).reshape(-1) if v_eps else (1 - lam) * v + lam * st["w"][2, p].double().cpu()
            close(st["v"][2, p], v, 1e-5)
        assert bool((st["k"][:2] == 0).all()) and bool((st["k"][2, :start] == 0).all()) and bool((st["v"][2, start + T:] == 0).all())
    with pytest.raises(ValueError):
        rope_kv_store(u.to(device), H * dk, G * dk, H, G, f.to(device), dims, st["k"], st["v"], sb, half, mag, v_eps=1e-3, v_first=(st["w"], lam))


def _dense(q, k, v, H, G, scale, cap, window, keep, start):
    """q [n, H, dk] at positions start.., keys and values of all positions so far: every score written out."""
    out = torch.zeros(q.shape[0], H, v.shape[-1], dtype=F64)
    for i in range(q.shape[0]):
        js = O.visible(start + i, {"size": window, "keep_first": keep})
        for h in range(H):
            g = h // (H // G)
            s = k[js, g] @ q[i, h] * scale
            s = cap * torch.tanh(s / cap) if cap else s
            out[i, h] = torch.softmax(s, 0) @ v[js, g]
    return out


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,dk,dv,bf16", [(4, 2, 6, 5, False), (4, 1, 16, 32, True), (3, 3, 48, 64, True), (4, 2, 64, 64, True), (2, 1, 96, 64, True),
                                            (4, 1, 128, 128, True), (2, 2, 192, 128, True), (2, 1, 24, 20, True)])
def test_kept_keys_behind_a_window(device, H, G, dk, dv, bf16):
    """The sweeps as an op: windows and kept runs below, at and above tiles of 32 keys, kept runs that reach into the
    window, a prompt, a portion that continues it, a decode step, one and several key splits; scalar and matrix-core
    sweeps, capped and not."""
    from llm_in_practise_amd.models.common import SeqBatch, SeqStateCache
    from llm_in_practise_amd.ops.attention import biased_attention
    g = torch.Generator().manual_seed(dk)
    n, dt = 150, torch.bfloat16 if bf16 else torch.float32
    q, k, v = ((1.5 * torch.randn(n, h, d, generator=g)).to(dt) for h, d in ((H, dk), (G, dk), (G, dv)))
    scale = 2.0 / math.sqrt(dk)
    for window, keep, cap in ((20, 4, 3.0), (33, 32, 0.0), (40, 70, 2.0), (1, 33, 5.0), (64, 1, 0.0), (500, 9, 3.0), (17, 0, 3.0)):
        cache = SeqStateCache([{"k": ((G * dk,), "kv"), "v": ((G * dv,), "kv")}], 3, 160, dt, device)
        st = cache.layers[0]
        st["k"].fill_(float("nan")), st["v"].fill_(float("nan"))               # what is not written must not be read ...
        st["k"][1, n:], st["v"][1, n:] = 0, 0                                    # (the end of the last tile is, and masked)
        st["k"][1, :n], st["v"][1, :n] = k.reshape(n, -1).to(device), v.reshape(n, -1).to(device)
        for a, e, splits in ((0, n, 1), (0, n, 3), (40, 93, 1), (97, 98, 1), (149, 150, 1), (149, 150, 7)):
            if device == "cpu" and splits > 1:
                continue
            sb = SeqBatch.packed(cache, [1], [e - a], [a])
            got = biased_attention(q[a:e].reshape(e - a, -1).to(device), st["k"], st["v"], None, H, G, scale, sb, window=window, nsplit=splits,
                                   softcap=cap, keep_first=keep)
            want = _dense(q[a:e].double(), k.double(), v.double(), H, G, scale, cap, window, keep, a).reshape(e - a, -1)
            assert err(got, want) < (2e-2 if bf16 else 2e-5), (window, keep, cap, a, e, splits)
    with pytest.raises(ValueError):
        biased_attention(q[:1].reshape(1, -1).to(device), st["k"], st["v"], None, H, G, scale, sb, keep_first=2)
    with pytest.raises(ValueError):
        biased_attention(q[:1].reshape(1, -1).to(device), st["k"], st["v"], None, H, G, scale, sb, block=8, window=4, keep_first=2)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kw", [dict(), dict(inner=1, state=1, dt_rank=1, conv=1), dict(inner=300, state=4, conv=2), dict(inner=33, state=8, conv=5),
                                dict(inner=40, state=16), dict(inner=130, state=12), dict(inner=28, state=32, dt_rank=9), dict(inner=19, state=33),
                                dict(inner=20, state=100), dict(inner=17, state=256)])
def test_selective_scan_alone(device, kw):
    """Register tilings of the scan from 1 to 256 states, channels that do and do not fill a block, one to five taps."""
    _check(device, [mamba(**kw), mamba(**kw)], decode_from=9, T=37)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("experts,top,shared,width", [(1, 1, 9, 44), (5, 1, 0, 44), (6, 2, 33, 45), (4, 4, 8, 44), (70, 3, 12, 44), (3, 2, 12, 42)])
def test_experts(device, experts, top, shared, width):
    """Top 1, some and all of the experts, without a shared one, with one of its own width and of the experts' (one more
    pair then); prompts on the pair path and (long ones) on the sorted path, rows of whole and cut 16-byte runs; a bias that
    only moved the choice would be seen."""
    cfg = config([mamba(mlp=moe(experts, top, 12, shared))], width=width)
    lm, W = build(cfg, device, 3)
    toks = tokens(90, cfg["vocab"], 4)
    want = logits_of(cfg, W, toks)
    close(replay(lm, 90, [([("a", toks)], ["a"])])["a"], want)
    close(replay(lm, 90, decoding(toks, 83))["a"], want)
    if top > 1:
        with planted(BIAS_CHOOSES_ONLY=True):
            assert err(logits_of(cfg, W, toks), want) > 1e-3
    h = torch.randn(700, width, generator=torch.Generator().manual_seed(1))                     # padded runs of rows
    from llm_in_practise_amd.models.common import SeqBatch, SeqStateCache
    sb = SeqBatch.packed(SeqStateCache([{}], 1, 700, torch.float32, device), [0], [700])
    close(lm.model.layers[0].ff(h.to(device), sb), O.experts(W, "l0.mlp.", cfg["layers"][0]["mlp"], h.double()))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("n,top,score", [(5, 2, "softmax"), (70, 3, "softmax"), (9, 9, "sigmoid")])
def test_router_bias(device, n, top, score):
    """A logit bias moves choice and weights, from given logits and from the fused product."""
    from llm_in_practise_amd.ops.moe import route_grouped, route_tokens
    g = torch.Generator().manual_seed(n)
    h, r, b = torch.randn(11, 24, generator=g), torch.randn(n, 24, generator=g), 3 * torch.randn(n, generator=g)
    z = h.double() @ r.double().t() + b.double()
    best = torch.topk(z, top, -1)
    s = torch.softmax(best.values, -1) if score == "softmax" else torch.sigmoid(best.values) / torch.sigmoid(best.values).sum(-1, keepdim=True)
    d = lambda t: t.to(device)      # noqa: E731
    for idx, w in (route_tokens(d(h), d(r), None, top, score=score, normalize=True, bias=d(b)),
                   route_grouped(d(h) @ d(r).t(), None, top, score=score, normalize=True, bias=d(b))):
        dense = torch.zeros(11, n, dtype=F64).scatter_(1, idx.long().cpu(), w.double().cpu())
        close(dense, torch.zeros(11, n, dtype=F64).scatter_(1, best.indices, s), 1e-4)
    idx2, w2 = route_tokens(d(h), d(r), None, top, score=score, normalize=True, bias=d(b), always=2)
    assert torch.equal(idx2[:, :top], route_tokens(d(h), d(r), None, top, score=score, normalize=True, bias=d(b))[0])
    assert idx2[:, top:].tolist() == [[n, n + 1]] * 11 and bool((w2[:, top:] == 1).all())
    with pytest.raises(ValueError):
        route_tokens(d(h), d(r), d(b), top, bias=d(b))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("W", [1, 36, 37, 600, 4100])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_residual_postnorm_op(device, W, dtype):
    """x + norm(y) in place and the copy or the next norm of it: widths with and without 16-byte rows and beyond a
    thread's registers, y as float or activations and as a column slice."""
    from llm_in_practise_amd.ops.norm import residual_postnorm
    g = torch.Generator().manual_seed(W)
    x, w, wn, wide = torch.randn(5, W, generator=g), torch.randn(W, generator=g), torch.randn(W, generator=g), 0.1 * torch.randn(5, W + 4, generator=g)
    for y in (wide[:, 4:], wide[:, 4:].to(dtype), wide.to(dtype)[:, 3:-1]):
        for nxt in (None, wn):
            xd = x.clone().to(device)
            dev_y = torch.empty(5, y.stride(0), dtype=y.dtype, device=device)[:, y.storage_offset():y.storage_offset() + W].copy_(y)
            h = residual_postnorm(xd, dev_y, w.to(device), 1e-3, dtype, None if nxt is None else nxt.to(device))
            want = x.double() + O.unit_rms(y.double(), 1e-3) * w.double()
            close(xd, want, 1e-5)
            close(h, want if nxt is None else O.unit_rms(want, 1e-3) * wn.double(), 1e-5 if dtype == torch.float32 else 1e-2)
            assert h.dtype == dtype and h.data_ptr() != xd.data_ptr()


@pytest.mark.parametrize("device", DEVICES)
def test_value_mixing(device):
    """Blend weights of 0, 1, negative; the first mixing layer is neither the first layer nor the first attention; layers
    between do not mix.  A blend with the mixing layer just before is seen, and so are the first one's values."""
    def tweak(W):
        W["l2.mix.vmix"], W["l4.mix.vmix"], W["l5.mix.vmix"] = (torch.tensor(x, dtype=F64) for x in (9.0, -0.7, 1.0))
    layers = [mamba(), att(v_mix=False, vdim=5, mlp=moe()), att(), att(v_mix=False, heads=2, kv_heads=2, vdim=3), att(size=4), att(heads=3, kv_heads=3, mlp=moe())]
    cfg, W, toks, want = _check(device, layers, decode_from=12, tweak=tweak)
    with planted(MIX_LAST=True):
        assert err(logits_of(cfg, W, toks), want) > 1e-3
    close(logits_of(cfg, {**W, "l2.mix.vmix": torch.tensor(0.0)}, toks), want, 1e-12)      # the first one's weight is not used
    assert TiburaxConfig.from_dict(cfg).value_source(5) == 2 and TiburaxConfig.from_dict(cfg).value_source(2) is None
    lm, _ = build(cfg, device, 1, tweak=tweak)
    close(replay(lm, 23, portions(toks, (2, 9, 2, 10)))["a"], want)


@pytest.mark.parametrize("device", DEVICES)
def test_state_carried_over_dirty_slot(device):
    """Pieces of 1-5 tokens, then of 60 and 40, into a slot that held another sequence: carried inputs, states and
    cached rows of the old sequence must not show; zeros before the start."""
    cfg = config([mamba(), att(size=30), mamba(conv=6, mlp=moe()), att(heads=3, kv_heads=3)])
    lm, W = build(cfg, device, 2)
    a, b = tokens(121, cfg["vocab"], 3), tokens(113, cfg["vocab"], 4)
    got = replay(lm, 128, [([("a", a)], ["a"])] + portions(b, (1, 3, 1, 5, 2, 1, 60, 40), "b"))
    close(got["b"], logits_of(cfg, W, b))


@pytest.mark.parametrize("device", DEVICES)
def test_residual_after_every_layer(device):
    """... which the norm must not have taken in."""
    cfg, W, toks, want = _check(device, BASE["layers"])
    with planted(NORM_OF_SUM=True):
        assert err(logits_of(cfg, W, toks), want) > 1e-2
    lm, _ = build(cfg, device, 1)
    lm.model.residual_tap = []
    lm(torch.tensor([toks], device=device))
    want = O.forward(cfg, W, toks)[1]
    assert len(lm.model.residual_tap) == len(want) == 5
    for got, w in zip(lm.model.residual_tap, want):
        close(got, w, 1e-4)


# ------------------------------------------------------------------------- schedules: cuts, batches, slots
@pytest.mark.parametrize("device", DEVICES)
def test_prefill_equals_token_by_token(device):
    lm, W = build(BASE, device, 5)
    toks = tokens(26, BASE["vocab"], 6)
    want = logits_of(BASE, W, toks)
    close(replay(lm, 26, [([("a", toks)], ["a"])])["a"], want)
    close(replay(lm, 26, [([("a", [t])], []) for t in toks])["a"], want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", [(2, 2, 2, 20), (7, 3, 2, 14), (1, 24, 1), (13, 13), (20, 2, 2, 2), (11, 11, 4), (33, 50, 2, 17), (64, 32, 16)])
def test_portions(device, cuts):
    """A prompt cut into portions (down to two tokens, at and off the kernels' 16- and 32-token runs) gives what the
    whole gives."""
    lm, W = build(BASE, device, 7)
    toks = tokens(sum(cuts), BASE["vocab"], 8)
    close(replay(lm, len(toks), portions(toks, cuts))["a"], logits_of(BASE, W, toks))


@pytest.mark.parametrize("device", DEVICES)
def test_unequal_batch_equals_each_alone(device):
    lm, W = build(BASE, device, 9)
    V = BASE["vocab"]
    reqs = {"a": tokens(1, V, 1) + tokens(9, V, 11), "b": tokens(50, V, 2), "c": tokens(12, V, 3), "d": tokens(2, V, 4)}
    first = {"a": 1, "b": 42, "c": 7, "d": 2}
    steps = [([(i, t[:first[i]]) for i, t in reqs.items()], ["d"])]
    for j in range(9):
        live = [(i, [t[first[i] + j]]) for i, t in reqs.items() if first[i] + j < len(t)]
        steps.append((live, [i for i, _ in live if first[i] + j + 1 == len(reqs[i])]))
    got = replay(lm, 120, steps)
    for i, t in reqs.items():
        close(got[i], logits_of(BASE, W, t)[:got[i].shape[0]])
        assert got[i].shape[0] == min(len(t), first[i] + 9)


@pytest.mark.parametrize("device", DEVICES)
def test_slots_freed_and_reused(device):
    """Requests pass through a pool of two slots one after another; a slot's old cache rows, states, carried inputs and
    positions must not reach its next sequence, shorter or longer."""
    lm, W = build(BASE, device, 12)
    V = BASE["vocab"]
    r = TraceRunner(lm, 64)
    r.engine = ServingEngine(lm, None, max_batch=2, max_model_len=65, use_graphs=False, start=False)
    for k, n in enumerate((31, 5, 18, 2, 40, 9)):
        t = tokens(n, V, 40 + n)
        cut = max(1, n - 3)
        a = r.step([{"id": f"r{k}", "tokens": t[:cut], "want": list(range(cut))}], [])
        parts = [a] + [r.step([{"id": f"r{k}", "tokens": [x], "want": [0]}], []) for x in t[cut:]]
        r.step([], [f"r{k}"])
        close(torch.cat(parts), logits_of(BASE, W, t))


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens_and_long_decoding(device):
    """Prompts of one, two and three tokens (fewer than the taps and the kept tokens), then 150 decoded tokens, past
    several windows."""
    cfg = config([mamba(mlp=moe()), att(size=13, keep=6, mlp=moe(4, 1)), att(size=40, keep=1)])
    lm, W = build(cfg, device, 13)
    for n in (1, 2, 3):
        toks = tokens(n, cfg["vocab"], n)
        close(replay(lm, 8, [([("a", toks)], ["a"])])["a"], logits_of(cfg, W, toks))
    toks = tokens(154, cfg["vocab"], 14)
    close(replay(lm, 160, decoding(toks, 4))["a"], logits_of(cfg, W, toks))


# ------------------------------------------- far keys, window edges, kept tokens, slow states: made to show
ASK, KEY = 0, 1   # queries of token ASK look for keys of token KEY; all other tokens are drawn from 2..


def _plant(dim, alpha=30.0):
    """The last (never rotated) entry of every query head is ``alpha`` times the input's component along ASK's embedding,
    that of every key head the same along KEY's, and no other embedding has such components: after the heads' norms an ASK
    query and a KEY key are nearly along that entry and score ``scale * dim``, all other pairs about nothing."""
    def tweak(W):
        E = W["embed"]
        ask = E[ASK] / E[ASK].norm()
        E[KEY] -= (E[KEY] @ ask) * ask
        key = E[KEY] / E[KEY].norm()
        E[2:] -= (E[2:] @ ask)[:, None] * ask + (E[2:] @ key)[:, None] * key
        W["l0.mix.q"][dim - 1::dim], W["l0.mix.k"][dim - 1::dim] = alpha * ask, alpha * key
    return tweak


def _marked(T, vocab, seed, asks, keys):
    toks = tokens(T, vocab, seed, lo=2)
    for p in asks:
        toks[p] = ASK
    for p in keys:
        toks[p] = KEY
    return toks


def _planted_model(device, size, keep, seed=17, **kw):
    cfg = config([att(heads=4, kv_heads=2, dim=10, vdim=8, rot=6, scale=2.0, cap=30.0, size=size, keep=keep, v_mix=False, mlp=moe())], **kw)
    lm, W = build(cfg, device, seed, tweak=_plant(10))
    return cfg, lm, W


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["window", "kept"])
def test_far_key_stands_out(device, kind):
    """An ASK query finds the one KEY key 650 positions back, inside a long window or among the kept tokens of a short
    one, over many tiles and, decoding, key splits; without that key the answer is another one."""
    at, (size, keep) = (30, (651, 0)) if kind == "window" else (36, (50, 37))
    cfg, lm, W = _planted_model(device, size, keep)
    T = 720
    toks = _marked(T, cfg["vocab"], 18, [680], [at])
    want = logits_of(cfg, W, toks)
    gone = list(toks)
    gone[at] = 2
    assert err(logits_of(cfg, W, gone)[680], want[680]) > 0.05
    with planted(**({"WINDOW_SHIFT": -1} if kind == "window" else {"KEEP_SHIFT": -1})):
        assert err(logits_of(cfg, W, toks)[680], want[680]) > 0.05
    close(replay(lm, 1400, [([("a", toks)], ["a"])])["a"], want)
    close(replay(lm, 1400, decoding(toks, 670))["a"], want)
    close(replay(lm, 1400, portions(toks, (31, 648, 2, 39)))["a"], want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size,keep", [(16, 4), (33, 1), (64, 32), (7, 40)])
def test_window_and_kept_edges(device, size, keep):
    """ASK queries whose KEY key is the oldest of the window, one older, the last kept token, the first that is not kept:
    in one prompt, decoded, and in portions cut at the asks.  Each edge one token off is seen at its ask."""
    cfg, lm, W = _planted_model(device, size, keep)
    b = keep + size + 5
    edges = {"win_in": (b + size - 1, b, dict(WINDOW_SHIFT=-1)), "win_out": (b + size, b, dict(WINDOW_SHIFT=1)),
             "keep_in": (b + size, keep - 1, dict(KEEP_SHIFT=-1)), "keep_out": (b + size, keep, dict(KEEP_SHIFT=1))}
    for ask, key, mistake in edges.values():
        T = ask + 6
        toks = _marked(T, cfg["vocab"], 16, [ask], [key])
        want = logits_of(cfg, W, toks)
        with planted(**mistake):
            assert err(logits_of(cfg, W, toks)[ask], want[ask]) > 0.05
        close(replay(lm, 2 * T, [([("a", toks)], ["a"])])["a"], want)
        close(replay(lm, 2 * T, decoding(toks, ask - 2))["a"], want)
        close(replay(lm, 2 * T, portions(toks, (ask - 1, 2, 5)))["a"], want)


@pytest.mark.parametrize("device", DEVICES)
def test_kept_tokens_keep_their_positions(device):
    """Kept tokens far behind the window are rotated and measured from where they stand, not as if moved up to it."""
    cfg = config([att(heads=4, kv_heads=2, dim=8, vdim=8, rot=8, base=50.0, scale=1.5, cap=20.0, size=10, keep=4, v_mix=False)])
    lm, W = build(cfg, device, 19)
    toks = tokens(60, cfg["vocab"], 20)
    want = logits_of(cfg, W, toks)
    with planted(KEPT_AT_EDGE=True):
        moved = logits_of(cfg, W, toks)
    assert err(moved[:10], want[:10]) < 1e-12 and err(moved[20:], want[20:]) > 0.01
    close(replay(lm, 64, decoding(toks, 33))["a"], want)


@pytest.mark.parametrize("device", DEVICES)
def test_slow_states_over_400_tokens(device):
    """States that keep nearly everything, so the last tokens depend on the first ones; they must survive prompt
    portions and 60 decode steps."""
    def tweak(W):
        for k in W:
            if k.endswith("A_log"):
                W[k] -= 6.0
            if k.endswith("dt.b"):
                W[k] -= 2.0
    cfg = config([mamba(mlp=moe())])
    lm, W = build(cfg, device, 21, tweak=tweak)
    toks = tokens(400, cfg["vocab"], 22)
    want = logits_of(cfg, W, toks)
    other = list(toks)
    other[3] = (toks[3] + 1) % cfg["vocab"]
    assert err(logits_of(cfg, W, other)[390:], want[390:]) > 1e-3
    steps = portions(toks[:340], (200, 140)) + [([("a", [t])], []) for t in toks[340:]]
    close(replay(lm, 400, steps)["a"], want, 5e-4)


# ---------------------------------------------------------------------------------- other sizes, bf16, files
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cfg", [
    config([att(heads=1, kv_heads=1, dim=1, vdim=1, rot=0, size=1, keep=0, mlp=moe(1, 1, 3, 1)), mamba(inner=1, state=1, dt_rank=1, conv=1),
            att(heads=1, kv_heads=1, dim=2, vdim=1, rot=2, size=2, keep=1)], width=6, vocab=5, scale=1.0),
    config([mamba(inner=35, state=11, dt_rank=2, conv=7, mlp=moe(11, 4, 9, 5)), att(heads=9, kv_heads=3, dim=10, vdim=7, rot=10, size=6, keep=2),
            att(heads=21, kv_heads=21, dim=5, vdim=1, rot=4, size=3, keep=5)], width=34, vocab=90, eps=1e-2, scale=0.5),
    config([att(heads=16, kv_heads=4, dim=4, vdim=9, rot=2, size=100, keep=3, cap=0, scaling=None), mamba(inner=70, state=20, dt_rank=5, conv=2)],
           width=21, vocab=33, scale=-2.0)])
def test_other_sizes(device, cfg):
    lm, W = build(cfg, device, 21)
    toks = tokens(19, cfg["vocab"], 22)
    close(replay(lm, 20, decoding(toks, 12))["a"], logits_of(cfg, W, toks))


ALL = moe(4, 4, 24, 16)     # every expert: no choice that bf16 rounding could turn


def _louder(W):
    """A norm on a sublayer's output blows up the rounding of an output that nearly cancels (an average over many values,
    say); a residual that starts larger keeps such a place from dominating the comparison."""
    W["embed"] *= 2


@pytest.mark.parametrize("device", DEVICES)
def test_bf16_weights_and_activations(device):
    cfg = copy.deepcopy(BASE)
    for lc in cfg["layers"]:
        if lc["mlp"]:
            lc["mlp"] = ALL
    lm, W = build(cfg, device, 23, dtype=torch.bfloat16, tweak=_louder)
    toks = tokens(24, cfg["vocab"], 24)
    close16(replay(lm, 24, decoding(toks, 15))["a"], logits_of(cfg, W, toks))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("heads,kv_heads", [(8, 2), (4, 4), (6, 2), (3, 1)])
@pytest.mark.parametrize("dim,vdim", [(16, 32), (48, 64), (64, 64), (96, 64), (96, 96), (128, 128), (192, 128)])
def test_bf16_matrix_core_sweeps(device, heads, kv_heads, dim, vdim):
    """Sizes the matrix-core sweeps take, in the forms for four heads per kv head, one head and grouped decode heads; 200
    tokens cross several whole and cut tiles of the window and of the kept run; decode with key splits."""
    mk = lambda size, keep: att(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, rot=dim // 2, scale=2.0 / dim ** 0.5, cap=9.0, size=size, keep=keep)      # noqa: E731
    cfg = config([mk(70, 5), mk(100, 70), mamba(inner=96, state=8, mlp=ALL)], width=64)
    lm, W = build(cfg, device, 33, dtype=torch.bfloat16, tweak=_louder)
    toks = tokens(200, cfg["vocab"], 34)
    want = logits_of(cfg, W, toks)
    close16(replay(lm, 400, decoding(toks, 185))["a"], want)
    close16(replay(lm, 400, portions(toks, (33, 64, 2, 101)))["a"], want)


@pytest.mark.parametrize("device", DEVICES)
def test_bf16_matrix_core_unequal_batch(device):
    """Prompts of 1, 40, 97 and 130 tokens packed into one step (tiles of one sequence never cross into the next),
    then decoded together, on sizes the matrix-core sweeps take."""
    cfg = config([att(heads=8, kv_heads=2, dim=32, vdim=32, rot=8, scale=0.15, cap=5.0, size=30, keep=9), mamba(inner=40, state=8, mlp=ALL),
                  att(heads=4, kv_heads=2, dim=16, vdim=32, rot=16, scale=0.2, size=64, keep=2, mlp=ALL)], width=64)
    lm, W = build(cfg, device, 29, dtype=torch.bfloat16, tweak=_louder)
    reqs = {i: tokens(n + 6, cfg["vocab"], 30 + n) for i, n in (("a", 1), ("b", 40), ("c", 97), ("d", 130))}
    steps = [([(i, t[:-6]) for i, t in reqs.items()], [])] + [([(i, [t[j - 6]]) for i, t in reqs.items()], []) for j in range(6)]
    got = replay(lm, 600, steps)
    for i, t in reqs.items():
        close16(got[i], logits_of(cfg, W, t))


def test_checkpoint_roundtrip_and_registry(tmp_path):
    from safetensors.torch import save_file
    from llm_in_practise_amd.models.registry import load_causal_lm
    W = {k: v.to(torch.bfloat16).contiguous() for k, v in weights(BASE, 9).items()}
    save_file(W, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(BASE))
    lm = load_causal_lm(str(tmp_path), dtype=torch.float32, device="cpu")
    assert type(lm).__name__ == "TiburaxForCausalLM" and lm.config.to_dict() == BASE
    toks = tokens(12, BASE["vocab"], 18)
    close(lm(torch.tensor([toks])).logits[0], logits_of(BASE, {k: v.double() for k, v in W.items()}, toks))
    for i, path, value in ((1, ("type",), "conv"), (0, ("mlp", "kind"), "dense"), (0, ("mixer", "kv_heads"), 4), (0, ("mlp", "router", "top"), 9),
                           (0, ("mixer", "mask", "size"), 0), (0, ("mixer", "mask", "keep_first"), -1), (0, ("mixer", "rot", "dims"), 3),
                           (0, ("mixer", "rot", "dims"), 12), (2, ("mixer", "vdim"), 6)):
        bad = copy.deepcopy(BASE)
        d = bad["layers"][i]
        for k in path[:-1]:
            d = d[k]
        d[path[-1]] = value
        with pytest.raises(ValueError):
            TiburaxConfig.from_dict(bad)
    del W["l0.mix.vmix"]                                            # never used
    TiburaxForCausalLM(TiburaxConfig.from_dict(BASE), W, torch.float32, "cpu")
    del W["l2.mix.vmix"]
    with pytest.raises(KeyError):
        TiburaxForCausalLM(TiburaxConfig.from_dict(BASE), W, torch.float32, "cpu")
    # the product's own random weights have every tensor the loader asks for
    lm = TiburaxForCausalLM.from_config(TiburaxConfig.from_dict(BASE), torch.float32, "cpu")
    assert lm(torch.tensor([toks])).logits.shape == (1, 12, BASE["vocab"])


def test_trace_replay_program(tmp_path):
    """``bin/trace_run`` as a user starts it: a checkpoint folder, JSON steps on standard input, one file of float
    logits per step that wants any, ``done <step>`` after every step."""
    import os
    import subprocess
    import numpy as np
    from safetensors.torch import save_file
    cfg = config([att(size=4), mamba(mlp=moe()), att()], width=40, vocab=53)
    W = {k: v.to(torch.bfloat16).contiguous() for k, v in weights(cfg, 5).items()}
    model, out = tmp_path / "model", tmp_path / "out"
    model.mkdir()
    save_file(W, str(model / "model.safetensors"))
    (model / "config.json").write_text(json.dumps(cfg))
    a, b = tokens(9, 53, 1), tokens(4, 53, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:7], "want": [0, 6]}, {"id": "b", "tokens": b[:3], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[7:8], "want": []}, {"id": "b", "tokens": b[3:], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[8:], "want": [0]}], "end": ["a"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    env = dict(os.environ, CUDA_VISIBLE_DEVICES="", HIP_VISIBLE_DEVICES="")
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(model), "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "16"], input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True,
                       text=True, timeout=600, env=env)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    W64 = {k: v.double() for k, v in W.items()}
    wa, wb = logits_of(cfg, W64, a), logits_of(cfg, W64, b)
    got = {n: torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, 53).copy()) for n in range(3)}
    close(got[0], wa[[0, 6]])
    close(got[1], wb[[3]])
    close(got[2], wa[[8]])


# ------------------------------------------------- greedy generation through the entry points and the scheduler
def _greedy(cfg, W, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(logits_of(cfg, W, seq)[-1].argmax()))
    return seq[len(prompt):]


class _Tok:
    """Token i <-> chr(0x100 + i): text in, text out, no special tokens."""
    eos_token_id = None
    pad_token_id = 0

    def encode(self, s, add_special_tokens=False):
        return [ord(c) - 0x100 for c in s]

    def decode(self, ids, skip_special_tokens=True):
        return "".join(chr(0x100 + int(i)) for i in ids)


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_engine_and_generate(device):
    cfg = config([att(size=5, keep=2, mlp=moe()), mamba(mlp=moe()), att()], width=40, vocab=53)
    lm, W = build(cfg, device, seed=10)
    prompts = [tokens(n, cfg["vocab"], 20 + n) for n in (9, 3, 14, 1, 6)]
    want = [_greedy(cfg, W, p, 7) for p in prompts]
    # generate(): right-padded batch of unequal prompts
    S = max(map(len, prompts))
    ids = torch.tensor([p + [0] * (S - len(p)) for p in prompts], device=device)
    mask = torch.tensor([[1] * len(p) + [0] * (S - len(p)) for p in prompts], device=device)
    out = lm.generate(ids, attention_mask=mask, max_new_tokens=7, do_sample=False)
    for b, p in enumerate(prompts):
        assert out[b, len(p):len(p) + 7].tolist() == want[b]
    # the serving engine: a queue, 3 slots for 5 requests (slots are reused), continuous batching; then chunked prefill:
    # long prompts enter 4 tokens per iteration between decode steps
    tok = _Tok()
    for slots, kw in ((3, {}), (2, {"chunked_prefill": 4})):
        eng = ServingEngine(lm, tok, max_batch=slots, max_model_len=64, use_graphs=False, **kw)
        try:
            reqs = [eng.submit(tok.decode(p), SamplingParams(max_tokens=7, temperature=0.0)) for p in prompts]
            for r, w in zip(reqs, want):
                while True:
                    kind, val = r.out.get(timeout=120)
                    if kind == "error":
                        raise RuntimeError(val)
                    if kind == "final":
                        break
                assert tok.encode(val["text"]) == w
        finally:
            eng.shutdown()


@pytest.mark.gpu
def test_decode_graphs_replay_equals_eager():
    """Captured decode steps, replayed many times with eager prefills between them, give the eager logits."""
    cfg = config([att(size=5, keep=2, mlp=moe()), mamba(mlp=moe()), att()], width=40, vocab=53)
    lm, W = build(cfg, "cuda", seed=11)
    V = cfg["vocab"]
    a, b, c = tokens(30, V, 30), tokens(12, V, 31), tokens(20, V, 32)

    def run(graphs):
        r, out = TraceRunner(lm, 200, use_graphs=graphs), {}
        steps = [([("a", a[:10]), ("b", b[:5])], [])] + [([("a", [a[10 + j]]), ("b", [b[5 + j]])], []) for j in range(7)]
        steps[-1] = (steps[-1][0], ["b"])
        steps += [([("c", c[:8])], [])] + [([("a", [a[17 + j]]), ("c", [c[8 + j]])], []) for j in range(12)]
        for entries, end in steps:
            got = r.step([{"id": i, "tokens": t, "want": list(range(len(t)))} for i, t in entries], end)
            o = 0
            for i, t in entries:
                out[i] = torch.cat([out[i], got[o:o + len(t)]]) if i in out else got[o:o + len(t)]
                o += len(t)
        return out
    eager, graph = run(False), run(True)
    for k in eager:
        close(graph[k], eager[k].double(), 1e-5)
    close(eager["a"], logits_of(cfg, W, a[:29]))
    close(eager["c"], logits_of(cfg, W, c))
