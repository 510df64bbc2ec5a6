"""Vefunex on the framework (packed batches, slot state, engine step functions, HIP kernels on a GPU) against the plain
float64 implementation of tests/vefunex_oracle.py.  Every test makes its own small configuration and weights; each
runs on the CPU path and, marked ``gpu``, on the HIP kernels."""
import copy
import json
import math

import pytest
import torch

import vefunex_oracle as O
from llm_in_practise_amd.infer.engine import SamplingParams, ServingEngine
from llm_in_practise_amd.infer.trace import TraceRunner
from llm_in_practise_amd.models.vefunex import VefunexConfig, VefunexForCausalLM

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F64 = torch.float64


def moe(experts=5, top=2, ff=20):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def att(heads=6, kv_heads=3, dim=8, vdim=10, coef=0.6, every=7, scale=0.4, mlp=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                                           "q_temp": {"coef": coef, "every": every}}, "mlp": mlp}


def par(heads=4, kv_heads=2, dim=10, vdim=6, rot=6, base=80.0, scale=0.5, cap=3.0, inner=26, state=5, dt_rank=3, conv=4,
        ls=1.3, rs=0.7, mlp=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": cap,
            "rot": {"base": base, "dims": rot}}
    right = {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": ls, "right_scale": rs}, "mlp": mlp}


def gla(heads=3, dim=6, vdim=9, tau=4.0, mlp=None):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "mlp": mlp}


def config(layers, width=48, vocab=61, eps=1e-5, taps=3, mult=0.45, cap=9.0):
    return {"architecture": "Vefunex", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps},
            "canon": {"taps": taps}, "residual_mult": mult, "logit_softcap": cap}


def weights(cfg, seed=0, rank=5):
    """Random float64 tensors under the checkpoint's names (``rank``: the gla decay's low rank)."""
    g = torch.Generator().manual_seed(seed)
    Wd, taps = cfg["width"], cfg["canon"]["taps"]

    def mat(o, i, s=1.0):
        return torch.randn(o, i, generator=g, dtype=F64) * s / math.sqrt(i)

    def vec(n, mean=1.0, s=0.2):
        return mean + s * torch.randn(n, generator=g, dtype=F64)
    W = {"embed": mat(cfg["vocab"], Wd, 0.8 * math.sqrt(Wd))}

    def norm(name):
        W.update({name: vec(Wd, 1.3), name + ".b": vec(Wd, 0.0), name + ".alpha": vec(1, 0.6, 0.1)[0]})

    def heads(q, m):
        H, G, dk, dv = (m[k] for k in ("heads", "kv_heads", "dim", "vdim"))
        W.update({q + "q": mat(H * dk, Wd, 1.6), q + "k": mat(G * dk, Wd, 1.6), q + "v": mat(G * dv, Wd), q + "o": mat(Wd, H * dv)})
    norm("final.norm")
    for i, lc in enumerate(cfg["layers"]):
        p, m, q = f"l{i}.", lc["mixer"], f"l{i}.mix."
        norm(p + "norm1")
        W[p + "canon1"] = 0.3 * torch.randn(Wd, taps, generator=g, dtype=F64)
        W[p + "dwa"] = torch.cat([vec(i + 1, 0.1, 0.3), vec(1, 0.9, 0.2)])
        if lc["type"] == "attention":
            heads(q, m)
        elif lc["type"] == "parallel":
            le, r, q2 = m["left"], m["right"], q + "right."
            heads(q + "left.", le)
            W[q + "left.g"], W[q + "left.sink"] = mat(le["heads"] * le["vdim"], Wd, 2.0), vec(le["heads"], 0.0, 1.0)
            n, N, R = r["inner"], r["state"], r["dt_rank"]
            W.update({q2 + "in": mat(2 * n, Wd), q2 + "conv": 0.5 * torch.randn(n, r["conv"], generator=g, dtype=F64),
                      q2 + "conv.b": vec(n, 0.0), q2 + "x": mat(R + 2 * N, n, 2.0), q2 + "dt": mat(n, R, 1.5),
                      q2 + "dt.b": vec(n, -1.0, 1.0), q2 + "A_log": vec(n * N, -0.5, 1.5).view(n, N), q2 + "D": vec(n),
                      q2 + "o": mat(Wd, n)})
        else:
            H, dk, dv = m["heads"], m["dim"], m["vdim"]
            W.update({q + "q": mat(H * dk, Wd, 1.5), q + "k": mat(H * dk, Wd, 1.5), q + "v": mat(H * dv, Wd), q + "g": mat(H * dv, Wd, 2.0),
                      q + "a1": mat(rank, Wd, 1.5), q + "a2": mat(H * dk, rank, 2.0), q + "a2.b": vec(H * dk, 1.0, 1.5),
                      q + "norm": vec(dv), q + "o": mat(Wd, H * dv)})
        mlp = lc.get("mlp")
        if mlp is not None:
            norm(p + "norm2")
            W[p + "canon2"] = 0.3 * torch.randn(Wd, taps, generator=g, dtype=F64)
            F_, q = mlp["expert"]["ff"], p + "mlp."
            W[q + "router"] = mat(mlp["router"]["experts"], Wd, 2.0)
            for e in range(mlp["router"]["experts"]):
                W.update({f"{q}e{e}.gate": mat(F_, Wd, 2.0), f"{q}e{e}.up": mat(F_, Wd, 2.0), f"{q}e{e}.down": mat(Wd, F_, 2.0)})
    return W


BASE = config([att(mlp=moe()), par(mlp=moe(7, 1, 12)), gla(), att(heads=4, kv_heads=4, dim=6, vdim=4, every=5, mlp=moe(3, 3, 8)),
               gla(heads=2, dim=5, vdim=4, tau=1.0, mlp=moe())])


def build(cfg, device, seed=0, dtype=torch.float32, tweak=None, **kw):
    W = weights(cfg, seed, **kw)
    if tweak:
        tweak(W)
    if dtype == torch.bfloat16:
        W = {k: v.to(torch.bfloat16).double() for k, v in W.items()}
    return VefunexForCausalLM(VefunexConfig.from_dict(cfg), W, dtype, device), W


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


def _check(device, layers, T=23, tweak=None, seed=1, decode_from=None, wkw=None, tol=2e-4, **kw):
    cfg = config(layers, **kw)
    lm, W = build(cfg, device, seed, tweak=tweak, **(wkw or {}))
    toks = tokens(T, cfg["vocab"], seed)
    want = logits_of(cfg, W, toks)
    close(replay(lm, T, [([("a", toks)], ["a"])])["a"], want, tol)
    if decode_from is not None:
        close(replay(lm, T, decoding(toks, decode_from))["a"], want, tol)
    return cfg, W, toks, want


def _silence(side):
    """One half of every parallel mixer gives nothing: its output projection is zero."""
    def tweak(W):
        for k in W:
            if k.endswith(f"mix.{side}.o"):
                W[k].zero_()
    return tweak


# --------------------------------------------------------------------------------------- each mechanism alone
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kw", [dict(), dict(heads=1, kv_heads=1, dim=2, vdim=3, every=1), dict(heads=5, kv_heads=5, dim=12, vdim=12, every=100),
                                dict(heads=8, kv_heads=2, dim=16, vdim=5, every=4, coef=-0.2), dict(heads=4, kv_heads=1, dim=6, vdim=32, every=2)])
def test_tempered_attention_alone(device, kw):
    """MHA, GQA and MQA, dim != vdim and equal, temperature steps of one position to beyond the sequence.  A key/value
    head read by the wrong query heads and a temperature one position late are seen by the oracle."""
    cfg, W, toks, want = _check(device, [att(**kw), att(**kw)], decode_from=9)
    m = cfg["layers"][0]["mixer"]
    if m["kv_heads"] > 1:
        with planted(KV_SHIFT=1):
            assert err(logits_of(cfg, W, toks), want) > 1e-2
    if m["q_temp"]["every"] < 20:
        with planted(TEMP_SHIFT=0):
            assert err(logits_of(cfg, W, toks), want) > 1e-3


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kw", [dict(), dict(heads=1, kv_heads=1, dim=4, vdim=4, rot=4, cap=0.5), dict(heads=5, kv_heads=5, dim=12, vdim=3, rot=0),
                                dict(heads=8, kv_heads=2, dim=16, vdim=32, rot=2, base=3.0, cap=40.0), dict(heads=4, kv_heads=1, dim=6, vdim=8, rot=6)])
def test_capped_attention_alone(device, kw):
    """The left half with the right half silenced: rotation of none, some and all dimensions, caps that bind and that
    do not, a sink per head, the output gate."""
    cfg, W, toks, want = _check(device, [par(**kw), par(**kw)], decode_from=9, tweak=_silence("right"))
    assert err(logits_of(cfg, {k: v * (3 if k.endswith("right.D") else 1) for k, v in W.items()}, toks), want) < 1e-12
    other = copy.deepcopy(cfg)
    for lc in other["layers"]:
        lc["mixer"]["left"]["softcap"] *= 1.5
    assert err(logits_of(other, W, toks), want) > (1e-3 if cfg["layers"][0]["mixer"]["left"]["softcap"] < 10 else 0.0)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kw", [dict(), dict(inner=1, state=1, dt_rank=1, conv=1), dict(inner=300, state=4, conv=2), dict(inner=33, state=8, conv=5),
                                dict(inner=40, state=16), dict(inner=130, state=12), dict(inner=24, state=32, dt_rank=9), dict(inner=19, state=33),
                                dict(inner=40, state=64), dict(inner=20, state=100), dict(inner=18, state=130), dict(inner=17, state=256)])
def test_selective_scan_alone(device, kw):
    """The right half with the left half silenced: every register tiling of the scan (1 to 256 states), channels that
    do and do not fill a block, one to five taps."""
    _check(device, [par(**kw), par(**kw)], decode_from=9, tweak=_silence("left"), T=37)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kw,rank", [(dict(), 5), (dict(heads=1, dim=1, vdim=1), 1), (dict(heads=2, dim=16, vdim=70, tau=16.0), 3),
                                     (dict(heads=1, dim=20, vdim=300, tau=0.5), 11), (dict(heads=4, dim=33, vdim=12), 2),
                                     (dict(heads=2, dim=64, vdim=64), 16), (dict(heads=1, dim=100, vdim=20), 20), (dict(heads=1, dim=200, vdim=9), 4)])
def test_gated_linear_attention_alone(device, kw, rank):
    """Every register tiling of the scan (key sizes 1 to 200), value sizes that do and do not fill a block, decay ranks
    1 to 20, tau below and above one."""
    _check(device, [gla(**kw), gla(**kw)], decode_from=9, wkw=dict(rank=rank), T=37)


@pytest.mark.parametrize("device", DEVICES)
def test_scan_ops_against_written_out_sums(device):
    """Both recurrences as ops over a dirty slot: outputs and the state they leave, strongly and hardly forgetting."""
    from llm_in_practise_amd.models.common import SeqBatch, SeqStateCache
    from llm_in_practise_amd.ops.recurrent import gated_linear_scan, selective_scan
    g = torch.Generator().manual_seed(5)
    T, H, dk, dv, C, N = 19, 2, 6, 5, 11, 7
    rnd = lambda *s: torch.randn(*s, generator=g)      # noqa: E731
    cache = SeqStateCache([{"S": ((H, dv, dk), "f32"), "R": ((C, N), "f32")}], 3, 64, torch.float32, device)
    to = lambda t: t.to(device)      # noqa: E731
    st = cache.layers[0]
    for t in st.values():
        t.fill_(7.0)                                           # a fresh sequence ignores what the slot held
    q, k, v, z, zb = rnd(T, H * dk), rnd(T, H * dk), rnd(T, H * dv), 8 * rnd(T, H * dk), rnd(H * dk)
    x, dtp, dtb, b, c, al, ds, zz = rnd(T, C), 3 * rnd(T, C), rnd(C), rnd(T, N), rnd(T, N), 2 * rnd(C, N), rnd(C), rnd(T, C)
    wide = torch.zeros(T, C + 4, device=device)
    got_o, got_y = [], []
    for a, e in ((0, 8), (8, 9), (9, 19)):                     # a prompt, one token, a continued portion
        sb = SeqBatch.packed(cache, [1], [e - a], [a])
        s = slice(a, e)
        got_o.append(gated_linear_scan(to(q[s]), to(k[s]), to(v[s]), to(z[s]), to(zb), 3.0, 0.25, st["S"], H, sb))
        got_y.append(selective_scan(to(x[s]), to(dtp[s]), to(dtb), to(b[s]), to(c[s]), to(al), to(ds), to(zz[s]), st["R"], sb,
                                    wide[s, 4:], 0.5))
    q, k, v, z, zb, x, dtp, dtb, b, c, al, ds, zz = (t.double() for t in (q, k, v, z, zb, x, dtp, dtb, b, c, al, ds, zz))
    got_o = torch.cat(got_o).cpu()
    for h in range(H):
        S = torch.zeros(dk, dv, dtype=F64)
        for t in range(T):
            r = slice(h * dk, (h + 1) * dk)
            S = (torch.sigmoid(z[t, r] + zb[r]) ** (1 / 3.0))[:, None] * S + torch.outer(k[t, r], v[t, h * dv:(h + 1) * dv])
            assert (got_o[t, h].double() - 0.25 * (S.t() @ q[t, r])).abs().max() < 1e-4
        close(st["S"][1, h].cpu(), S.t(), 1e-5)
    S = torch.zeros(C, N, dtype=F64)
    for t in range(T):
        dt = torch.log1p(torch.exp(dtp[t] + dtb))
        S = torch.exp(-dt[:, None] * torch.exp(al)) * S + (dt * x[t])[:, None] * b[t][None]
        y = 0.5 * (S @ c[t] + ds * x[t]) * zz[t] * torch.sigmoid(zz[t])
        assert (torch.cat(got_y)[t].cpu().double() - y).abs().max() < 1e-4
    close(st["R"][1].cpu(), S, 1e-5)
    assert bool((wide[:, :4] == 0).all()) and bool((st["R"][0] == 7).all()) and bool((st["S"][2] == 7).all())


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("taps", [0, 1, 2, 3, 4, 5, 8])
@pytest.mark.parametrize("W", [36, 37, 600])
def test_residual_dyt_op(device, taps, W):
    """Weighted add, average over depth, Dynamic Tanh and input convolution against the formulas: widths with and
    without 16-byte rows, runs longer than a block's, pieces from 1 to 70 tokens into a dirty slot, a packed second
    sequence, a row whose state must not change."""
    from llm_in_practise_amd.models.common import SeqBatch, SeqStateCache
    from llm_in_practise_amd.ops.norm import residual_dyt
    g = torch.Generator().manual_seed(3)
    n, alpha, mult = 3, 0.7, -0.4
    rnd = lambda *s: torch.randn(*s, generator=g)      # noqa: E731
    T, T2 = 150, 41
    w, b, depth = rnd(W), rnd(W), rnd(n + 1)
    conv = rnd(taps, W) if taps else None
    to = lambda t: None if t is None else t.to(device)      # noqa: E731
    data = {i: (rnd(m, W), rnd(m, W), rnd(5, m, W)) for i, m in ((0, T), (2, T2))}
    spec = {"c": ((taps - 1, W), "f32")} if taps > 1 else {}
    cache = SeqStateCache([spec], 4, 400, torch.float32, device)
    if spec:
        cache.layers[0]["c"].fill_(9.0)
    got = {0: [], 2: []}
    cuts = [({0: 33, 2: 1}), ({0: 1, 2: 40}), ({0: 2}), ({0: 70}), ({0: 5}), ({0: 39})]
    at = {0: 0, 2: 0}
    for cut in cuts:
        slots = sorted(cut)
        sb = SeqBatch.packed(cache, slots, [cut[s] for s in slots], [at[s] for s in slots])
        pick = lambda j: torch.cat([data[s][j][..., at[s]:at[s] + cut[s], :] for s in slots], -2)      # noqa: E731
        streams = to(pick(2))
        r, h = residual_dyt(to(pick(0)), to(pick(1)), mult, to(w), to(b), alpha, torch.float32, to(conv), cache.layers[0].get("c"),
                            streams, n, to(depth), sb)
        o = 0
        for s in slots:
            got[s].append((r[o:o + cut[s]].cpu(), h[o:o + cut[s]].cpu(), streams[n, o:o + cut[s]].cpu()))
            o += cut[s]
            at[s] += cut[s]
    for s in (0, 2):
        x, y, st = (t.double() for t in data[s])
        new = x + mult * y
        r = sum(depth[j].double() * st[j] for j in range(n)) + depth[n].double() * new
        h = torch.tanh(alpha * r) * w.double() + b.double()
        if taps:
            h = h + O.causal_conv(h, conv.double().t())
        for j, want in enumerate((r, h, new)):
            close(torch.cat([p[j] for p in got[s]]), want, 1e-5)
    if spec:
        assert bool((cache.layers[0]["c"][1] == 9).all()) and bool((cache.layers[0]["c"][3] == 9).all())
    # a decode row that is not live leaves its slot alone; no sublayer output and no average: the residual passes through
    cache.pos.fill_(5)
    if spec:
        cache.layers[0]["c"].fill_(2.0)
    cache.set_live([1], 3)
    x = rnd(3, W).to(device)
    r, h = residual_dyt(x, None, 1.0, to(w), to(b), alpha, torch.float32, to(conv), cache.layers[0].get("c"), None, 0, None,
                        SeqBatch.decoding(cache, 3))
    assert torch.equal(r, x)
    hv = torch.tanh(alpha * x.double().cpu()) * w.double() + b.double()
    want = hv + (conv[-1].double() * hv + 2.0 * conv[:-1].double().sum(0) if taps else 0.0)
    close(h[1:2], want[1:2], 1e-5)
    if spec:
        c = cache.layers[0]["c"].cpu().double()
        assert bool((c[0] == 2).all()) and bool((c[2] == 2).all())
        close(c[1, -1], hv[1], 1e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("experts,top", [(1, 1), (5, 1), (6, 2), (4, 4), (70, 3)])
def test_experts(device, experts, top):
    """Top 1, some and all of the experts; prompts on the pair path and (long ones) on the sorted path; the score
    multiplies the expert's input."""
    cfg = config([gla(mlp=moe(experts, top, 12))])
    lm, W = build(cfg, device, 3)
    toks = tokens(90, cfg["vocab"], 4)
    want = logits_of(cfg, W, toks)
    close(replay(lm, 90, [([("a", toks)], ["a"])])["a"], want)
    close(replay(lm, 90, decoding(toks, 83))["a"], want)
    from llm_in_practise_amd.ops.moe import moe_glu_experts, route_tokens
    h = torch.randn(700, 48, generator=torch.Generator().manual_seed(1)).to(device)          # padded runs of rows
    ff = lm.model.layers[0].ff
    idx, w = route_tokens(h, ff.router, None, top, score="sigmoid")
    got = moe_glu_experts(h, ff.w_gu, ff.w_d, idx, w, 0.0, None, False, act="silu", weight_input=True)
    close(got, O.experts(W, "l0.mlp.", cfg["layers"][0]["mlp"], h.double().cpu()))
    assert err(moe_glu_experts(h, ff.w_gu, ff.w_d, idx, w, 0.0, None, False, act="silu"), got.double().cpu()) > 1e-2


@pytest.mark.parametrize("device", DEVICES)
def test_value_norm_temperature_and_rotation_on_a_cache(device):
    """rope_kv_store with every part at once: rotated q times the temperature, rotated k, unit-RMS values, at positions
    on both sides of temperature steps."""
    from llm_in_practise_amd.models.common import SeqBatch, SeqStateCache
    from llm_in_practise_amd.ops.attention import rope_kv_store, rotary_inv_freq
    H, G, dk, dv, dims, T = 4, 2, 10, 70, 6, 9
    u = torch.randn(T, (H + G) * dk + G * dv, generator=torch.Generator().manual_seed(1))
    for start in (0, 15, 4094):
        cache = SeqStateCache([{"k": ((G * dk,), "kv"), "v": ((G * dv,), "kv")}], 3, 4200, torch.float32, device)
        sb, st = SeqBatch.packed(cache, [2], [T], [start]), cache.layers[0]
        q = rope_kv_store(u.to(device), H * dk, G * dk, H, G, rotary_inv_freq(dims, 30.0).to(device), dims, st["k"], st["v"], sb,
                          half=False, temp=(0.7, 8), v_eps=1e-3)
        for t in range(T):
            p = start + t
            for h in range(H + G):
                want = O.rotate_neighbours(u[t, h * dk:(h + 1) * dk].double(), p, dims, 30.0)
                got = q[t, h * dk:(h + 1) * dk] if h < H else st["k"][2, p, (h - H) * dk:(h - H + 1) * dk]
                close(got, want * (O.temperature(p, 0.7, 8) if h < H else 1.0), 1e-3 if start > 4000 else 1e-5)
            for h in range(G):
                want = O.unit_rms(u[t, (H + G) * dk + h * dv:][:dv].double(), 1e-3)
                close(st["v"][2, p, h * dv:(h + 1) * dv], want, 1e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("taps", [1, 2, 5, 8])
def test_input_convolutions(device, taps):
    """One tap (the current input only) to more taps than some prompts have tokens; both sublayers' convolutions."""
    cfg, W, toks, want = _check(device, [par(mlp=moe()), gla(mlp=moe())], taps=taps, decode_from=2)
    for name in ("l1.canon1", "l0.canon2"):
        assert err(logits_of(cfg, {**W, name: W[name] * 0}, toks), want) > 1e-3


@pytest.mark.parametrize("device", DEVICES)
def test_state_carried_over_dirty_slot(device):
    """Pieces of 1-5 tokens, then of 60 and 40, into a slot that held another sequence: carried inputs, states and
    cached rows of the old sequence must not show; zeros before the start."""
    cfg = config([par(), att(), gla(mlp=moe())], taps=4)
    lm, W = build(cfg, device, 2)
    a, b = tokens(121, cfg["vocab"], 3), tokens(113, cfg["vocab"], 4)
    got = replay(lm, 128, [([("a", a)], ["a"])] + portions(b, (1, 3, 1, 5, 2, 1, 60, 40), "b"))
    close(got["b"], logits_of(cfg, W, b))


@pytest.mark.parametrize("device", DEVICES)
def test_residual_after_every_layer(device):
    cfg, W, toks, _ = _check(device, BASE["layers"])
    lm, _ = build(cfg, device, 1)
    lm.model.residual_tap = []
    lm(torch.tensor([toks], device=device))
    want = O.forward(cfg, W, toks)[1]
    assert len(lm.model.residual_tap) == len(want) == 5
    for got, w in zip(lm.model.residual_tap, want):
        close(got, w, 1e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_branch_weights_depth_weights_and_bounds(device):
    """Branch weights of 0 and -1, a layer that forgets its own result and looks at the embedding, a large and a
    negative residual weight, a tight bound on the logits."""
    def tweak(W):
        W["l1.dwa"] = torch.tensor([1.5, -0.7, 0.0], dtype=F64)
    for mult, cap in ((2.0, 1.0), (-0.5, 50.0)):
        cfg, W, toks, want = _check(device, [par(ls=0.0, rs=2.5), gla(mlp=moe()), par(ls=-1.0, rs=1.0, mlp=moe())], decode_from=12,
                                    tweak=tweak, mult=mult, cap=cap)
        assert want.abs().max() <= cap
        other = copy.deepcopy(cfg)
        other["layers"][2]["mixer"]["left_scale"] = 1.0
        assert err(logits_of(other, W, toks), want) > 1e-3


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
    """Prompts of one, two and three tokens (fewer than the taps), then 150 decoded tokens."""
    cfg = config([par(mlp=moe()), att(every=13), gla(mlp=moe(4, 1))], taps=4)
    lm, W = build(cfg, device, 13)
    for n in (1, 2, 3):
        toks = tokens(n, cfg["vocab"], n)
        close(replay(lm, 8, [([("a", toks)], ["a"])])["a"], logits_of(cfg, W, toks))
    toks = tokens(154, cfg["vocab"], 14)
    close(replay(lm, 160, decoding(toks, 4))["a"], logits_of(cfg, W, toks))


# ------------------------------------------- far keys, temperature steps, sinks, slow forgetting: made to show
ASK, KEY = 0, 1   # queries of token ASK look for keys of token KEY; all other tokens are drawn from 2..


def _plant(prefix, dim, alpha):
    """In the last (never rotated) dimension of every head, queries get ``alpha`` times the input's component along
    ASK's embedding and keys the same along KEY's: an ASK query gives nearly all its weight to a KEY key."""
    def tweak(W):
        for n, tok in (("q", ASK), ("k", KEY)):
            e = W["embed"][tok] / W["embed"][tok].norm()
            W[f"l0.mix.{prefix}{n}"][dim - 1::dim] += alpha * e
    return tweak


def _marked(T, vocab, seed, asks, keys):
    toks = tokens(T, vocab, seed, lo=2)
    for p in asks:
        toks[p] = ASK
    for p in keys:
        toks[p] = KEY
    return toks


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["attention", "left"])
def test_far_key_stands_out(device, kind):
    """An ASK query finds the one KEY key 650 positions back, over many tiles and, decoding, key splits; without that
    key, or with a memory of 649 positions, the answer is another one."""
    if kind == "attention":
        cfg, tweak = config([att(heads=4, kv_heads=2, dim=8, vdim=8, every=64, mlp=moe())]), _plant("", 8, 5.0)
    else:
        cfg = config([par(heads=4, kv_heads=2, dim=8, vdim=8, rot=4, base=1e6, cap=40.0, ls=2.0, rs=0.3, mlp=moe())])
        tweak = _plant("left.", 8, 4.0)
    T = 720
    toks = _marked(T, cfg["vocab"], 18, [680], [30])
    lm, W = build(cfg, device, 17, tweak=tweak)
    want = logits_of(cfg, W, toks)
    gone = list(toks)
    gone[30] = 2
    assert err(logits_of(cfg, W, gone)[680], want[680]) > 0.05
    with planted(FAR_LIMIT=650):
        assert err(logits_of(cfg, W, toks)[680], want[680]) > 0.05
    close(replay(lm, 1400, [([("a", toks)], ["a"])])["a"], want)
    close(replay(lm, 1400, decoding(toks, 670))["a"], want)
    close(replay(lm, 1400, portions(toks, (31, 648, 2, 39)))["a"], want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("every", [1, 16, 33])
def test_temperature_steps(device, every):
    """A query temperature that jumps at every step: positions just before, at and after a step, in a prompt, decoded,
    and in portions cut at the steps.  The oracle one position late differs widely at the step and only there."""
    cfg = config([att(coef=3.0, every=every, scale=0.3, mlp=moe())])
    lm, W = build(cfg, device, 15)
    T = 2 * every + 9
    toks = tokens(T, cfg["vocab"], 16)
    want = logits_of(cfg, W, toks)
    with planted(TEMP_SHIFT=0):
        late = logits_of(cfg, W, toks)
    assert err(late[2 * every - 1], want[2 * every - 1]) > 0.01
    if every > 1:
        assert err(late[:every - 1], want[:every - 1]) < 1e-12
    close(replay(lm, T, [([("a", toks)], ["a"])])["a"], want)
    close(replay(lm, T, decoding(toks, max(1, every - 2)))["a"], want)
    if every > 1:
        close(replay(lm, T, portions(toks, (every - 1, 2, every - 2, 2, 8)))["a"], want)


@pytest.mark.parametrize("device", DEVICES)
def test_sinks_take_their_share(device):
    """Sink scores far above the keys' scores (and the cap): they hold most of every softmax, each head its own."""
    def tweak(W):
        W["l0.mix.left.sink"] = torch.tensor([6.0, 1.0, 4.0, -3.0], dtype=F64)
    cfg = config([par(scale=0.05, cap=2.0, ls=2.0, rs=0.3, mlp=moe())])
    lm, W = build(cfg, device, 19, tweak=tweak)
    toks = tokens(30, cfg["vocab"], 20)
    want = logits_of(cfg, W, toks)
    with planted(USE_SINK=False):
        assert err(logits_of(cfg, W, toks), want) > 0.05
    W2 = dict(W)
    W2["l0.mix.left.sink"] = torch.tensor([4.0, 1.0, 6.0, -3.0], dtype=F64)
    assert err(logits_of(cfg, W2, toks), want) > 1e-3               # per head, not one number
    close(replay(lm, 32, decoding(toks, 17))["a"], want)
    close(replay(lm, 600, decoding(toks, 17))["a"], want)           # the sink counts once over several key splits


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["scan", "gla"])
def test_slow_states_over_400_tokens(device, kind):
    """States that keep nearly everything, so the last tokens depend on the first ones; they must survive prompt
    portions and 60 decode steps."""
    def tweak(W):
        for k in W:
            if k.endswith("a2.b"):
                W[k] += 9.0
            if k.endswith("A_log"):
                W[k] -= 6.0
            if k.endswith("dt.b"):
                W[k] -= 2.0
    layer = gla(heads=2, dim=12, vdim=10, mlp=moe()) if kind == "gla" else par(ls=0.2, rs=1.5, mlp=moe())
    cfg = config([layer])
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
    config([att(heads=1, kv_heads=1, dim=1, vdim=1, every=1, mlp=moe(1, 1, 3)), gla(heads=1, dim=1, vdim=1),
            par(heads=1, kv_heads=1, dim=2, vdim=1, rot=2, inner=1, state=1, dt_rank=1, conv=1, ls=1.0, rs=1.0)], width=6, vocab=5, taps=1, mult=1.0),
    config([par(heads=9, kv_heads=3, dim=10, vdim=7, rot=10, inner=35, state=11, dt_rank=2, conv=7, mlp=moe(11, 4, 9)),
            att(heads=7, kv_heads=7, dim=5, vdim=3)], width=34, vocab=90, eps=1e-3, taps=6),
    config([gla(heads=7, dim=3, vdim=17, tau=30.0, mlp=moe(3, 1, 5)), gla(heads=1, dim=17, vdim=2), att(heads=16, kv_heads=4, dim=4, vdim=9)],
           width=21, vocab=33, taps=2)])
def test_other_sizes(device, cfg):
    lm, W = build(cfg, device, 21, rank=2)
    toks = tokens(19, cfg["vocab"], 22)
    close(replay(lm, 20, decoding(toks, 12))["a"], logits_of(cfg, W, toks))


ALL = moe(4, 4, 24)     # every expert: no choice that bf16 rounding could turn


@pytest.mark.parametrize("device", DEVICES)
def test_bf16_weights_and_activations(device):
    cfg = copy.deepcopy(BASE)
    cfg["residual_mult"] = 0.2
    for lc in cfg["layers"]:
        if lc["mlp"]:
            lc["mlp"] = ALL
    lm, W = build(cfg, device, 23, dtype=torch.bfloat16)
    toks = tokens(24, cfg["vocab"], 24)
    close16(replay(lm, 24, decoding(toks, 15))["a"], logits_of(cfg, W, toks))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("heads,kv_heads", [(8, 2), (4, 4), (6, 2), (3, 1)])
def test_bf16_matrix_core_sizes_long_context(device, heads, kv_heads):
    """Sizes the matrix-core sweeps take (four heads per kv head, one, three; narrow and wide instantiations), 300 keys,
    decode with key splits, gate and cap in the sweep and in the merge of the splits."""
    cfg = config([att(heads=heads, kv_heads=kv_heads, dim=32, vdim=64, every=50, scale=0.15, mlp=ALL),
                  par(heads=heads, kv_heads=kv_heads, dim=48, vdim=32, rot=16, scale=0.12, cap=4.0, inner=64, state=16, dt_rank=8),
                  gla(heads=2, dim=32, vdim=32),
                  par(heads=heads, kv_heads=kv_heads, dim=96, vdim=96, rot=96, scale=0.1, cap=6.0, inner=48, state=32, dt_rank=4, mlp=ALL)],
                 width=64, mult=0.2)
    lm, W = build(cfg, device, 25, dtype=torch.bfloat16)
    toks = tokens(300, cfg["vocab"], 26)
    close16(replay(lm, 600, decoding(toks, 290))["a"], logits_of(cfg, W, toks))


@pytest.mark.parametrize("device", DEVICES)
def test_bf16_matrix_core_unequal_batch(device):
    """Prompts of 1, 40, 97 and 130 tokens packed into one step (tiles of one sequence never cross into the next),
    then decoded together, on sizes the matrix-core sweeps take."""
    cfg = config([par(heads=8, kv_heads=2, dim=32, vdim=32, rot=8, scale=0.15, cap=5.0, inner=40, state=8, mlp=ALL),
                  att(heads=4, kv_heads=2, dim=16, vdim=32, every=20, scale=0.2), gla(heads=2, dim=24, vdim=16, mlp=ALL)], width=64, mult=0.2)
    lm, W = build(cfg, device, 29, dtype=torch.bfloat16)
    reqs = {i: tokens(n + 6, cfg["vocab"], 30 + n) for i, n in (("a", 1), ("b", 40), ("c", 97), ("d", 130))}
    steps = [([(i, t[:-6]) for i, t in reqs.items()], [])] + [([(i, [t[j - 6]]) for i, t in reqs.items()], []) for j in range(6)]
    got = replay(lm, 600, steps)
    for i, t in reqs.items():
        close16(got[i], logits_of(cfg, W, t))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("heads,kv_heads", [(4, 1), (3, 3), (6, 2)])
@pytest.mark.parametrize("dim", [64, 96, 128])
def test_bf16_exact_size_sweeps(device, dim, heads, kv_heads):
    """Head sizes with a sweep of their own (64, 96, 128), with and without bounded scores, in the forms for four heads
    per kv head, one head and grouped decode heads; 200 tokens cross several whole and cut tiles."""
    cfg = config([att(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, every=40, scale=0.8 / dim ** 0.5),
                  par(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, rot=dim // 2, scale=1.2 / dim ** 0.5, cap=2.5, inner=24, state=8,
                      mlp=ALL)], width=64, mult=0.2)
    lm, W = build(cfg, device, 33, dtype=torch.bfloat16)
    toks = tokens(200, cfg["vocab"], 34)
    want = logits_of(cfg, W, toks)
    close16(replay(lm, 400, decoding(toks, 185))["a"], want)
    close16(replay(lm, 400, portions(toks, (33, 64, 2, 101)))["a"], want)


@pytest.mark.parametrize("device", DEVICES)
def test_bf16_wide_heads(device):
    """Heads of 128, 160 and 256 columns (the sweeps' wide instantiations), key size 128 in the linear attention."""
    cfg = config([att(heads=4, kv_heads=1, dim=128, vdim=128, every=30, scale=0.06, mlp=ALL), gla(heads=1, dim=128, vdim=64),
                  par(heads=2, kv_heads=1, dim=160, vdim=256, rot=32, scale=0.06, cap=5.0, inner=70, state=64, mlp=ALL)], width=64, mult=0.2)
    lm, W = build(cfg, device, 27, dtype=torch.bfloat16)
    toks = tokens(150, cfg["vocab"], 28)
    close16(replay(lm, 300, decoding(toks, 140))["a"], logits_of(cfg, W, toks))


def test_checkpoint_roundtrip_and_registry(tmp_path):
    from safetensors.torch import save_file
    from llm_in_practise_amd.models.registry import load_causal_lm
    W = {k: v.to(torch.bfloat16).contiguous() for k, v in weights(BASE, 9).items()}
    save_file(W, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(BASE))
    lm = load_causal_lm(str(tmp_path), dtype=torch.float32, device="cpu")
    assert type(lm).__name__ == "VefunexForCausalLM" and lm.config.to_dict() == BASE
    assert lm.lm_head.weight.data_ptr() == lm.model.embed_tokens.data_ptr()
    toks = tokens(12, BASE["vocab"], 18)
    close(lm(torch.tensor([toks])).logits[0], logits_of(BASE, {k: v.double() for k, v in W.items()}, toks))
    for i, path, value in ((0, ("type",), "conv"), (0, ("mlp", "kind"), "dense"), (0, ("mixer", "kv_heads"), 4), (0, ("mlp", "router", "top"), 9),
                           (0, ("mixer", "q_temp", "every"), 2.5), (1, ("mixer", "left", "rot", "dims"), 3), (1, ("mixer", "left", "rot", "dims"), 12)):
        bad = copy.deepcopy(BASE)
        d = bad["layers"][i]
        for k in path[:-1]:
            d = d[k]
        d[path[-1]] = value
        with pytest.raises(ValueError):
            VefunexConfig.from_dict(bad)
    with pytest.raises(ValueError):                                # depth weights of another layer count
        VefunexForCausalLM(VefunexConfig.from_dict(BASE), {**W, "l2.dwa": W["l1.dwa"]}, torch.float32, "cpu")
    del W["l1.mix.left.sink"]
    with pytest.raises(KeyError):
        VefunexForCausalLM(VefunexConfig.from_dict(BASE), W, torch.float32, "cpu")
    # the product's own random weights have every tensor the loader asks for
    lm = VefunexForCausalLM.from_config(VefunexConfig.from_dict(BASE), torch.float32, "cpu")
    assert lm(torch.tensor([toks])).logits.shape == (1, 12, BASE["vocab"])


def test_trace_replay_program(tmp_path):
    """``bin/trace_run`` as a user starts it: a checkpoint folder, JSON steps on standard input, one file of float
    logits per step that wants any, ``done <step>`` after every step."""
    import os
    import subprocess
    import numpy as np
    from safetensors.torch import save_file
    cfg = config([par(mlp=moe()), att(), gla()], width=40, vocab=53)
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
    cfg = config([par(mlp=moe()), gla(mlp=moe()), att(every=5)], width=40, vocab=53)
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
    cfg = config([par(mlp=moe()), gla(mlp=moe()), att(every=5)], width=40, vocab=53)
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


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("T,K,C", [(1, 1, 1), (3, 12, 130), (8, 16, 64), (9, 128, 200), (64, 256, 65), (65, 40, 70), (5, 300, 33)])
def test_float_products_of_low_rank(device, T, K, C):
    """matmul_f32 on column slices of bf16 rows: few and many rows, odd ranks and widths."""
    from llm_in_practise_amd.ops.gemm import matmul_f32
    g = torch.Generator().manual_seed(K)
    wide, w = torch.randn(T, K + 11, generator=g).to(torch.bfloat16), torch.randn(C, K, generator=g).to(torch.bfloat16)
    got = matmul_f32(wide.to(device)[:, 3:3 + K], w.to(device))
    assert got.dtype == torch.float32
    close(got, wide[:, 3:3 + K].double() @ w.double().t(), 1e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dv", [4, 20, 36, 64, 100, 128, 200, 256, 300, 7])
def test_head_norm_and_gate_read_out(device, dv):
    """Per-head RMS norm with a shared or per-head weight, sigmoid and SiLU gates, into a scaled column slice."""
    from llm_in_practise_amd.ops.norm import head_norm_gate
    g = torch.Generator().manual_seed(dv)
    T, H = 5, 3
    o, wide = torch.randn(T, H, dv, generator=g), torch.randn(T, H * dv + 8, generator=g)
    gate = wide[:, 8:]
    for act, w in (("sigmoid", torch.randn(dv, generator=g)), ("silu", torch.randn(H * dv, generator=g))):
        z = gate.double()
        want = O.unit_rms(o.double(), 1e-5) * (w.double() if w.numel() == dv else w.double().view(H, dv))
        want = want.reshape(T, -1) * (torch.sigmoid(z) if act == "sigmoid" else O.silu(z))
        close(head_norm_gate(o.to(device), w.to(device), wide.to(device)[:, 8:], 1e-5, act=act), want, 1e-5)
        out = torch.zeros(T, H * dv + 4, device=device)
        head_norm_gate(o.to(device), w.to(device), wide.to(device)[:, 8:], 1e-5, out=out[:, 4:], scale=-0.3, act=act)
        close(out[:, 4:], -0.3 * want, 1e-5)
        assert bool((out[:, :4] == 0).all())
