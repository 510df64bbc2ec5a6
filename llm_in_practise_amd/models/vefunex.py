"""Vefunex: a pre-normed decoder whose layers read an average over depth, with attention, selective-scan and
gated-linear-attention mixers and routed feed-forwards.

* every norm is a Dynamic Tanh: ``tanh(alpha x) * w + b`` per channel, with a learned scalar ``alpha`` and no statistics;
* what a sublayer reads is the normed residual plus a short causal convolution of itself over time, per channel
  (``canon1`` before the mixer, ``canon2`` before the feed-forward); the last ``taps - 1`` normed inputs of both are part
  of a sequence's state in every layer;
* a sublayer's output is added with one fixed weight (``residual_mult``); after every layer the residual becomes a
  learned weighted sum of the embedding output and all layer results so far;
* ``attention`` mixers: grouped-query attention without rotation; queries get warmer with the position in steps
  (``1 + coef ln(floor((p + 1) / every) + 1)``), every head's value has unit root mean square;
* ``parallel`` mixers: two mixers read the same input and their outputs are added with fixed weights.  Left:
  grouped-query attention with rotation of neighbouring pairs in the first ``rot.dims`` entries of each head, scores
  bounded by ``softcap``, a learned sink score per head and an element-wise sigmoid output gate.  Right: a selective
  state space (short convolution + SiLU, step size per channel, decay per channel and state, SiLU gate);
* ``gla`` mixers: gated linear attention, a ``[dim, vdim]`` matrix per head whose rows decay by
  ``sigmoid(z)^(1 / tau)`` with a low-rank ``z``; the read-out is RMS-normed per head and gated by a SiLU;
* feed-forwards: SiLU-GLU experts chosen by sigmoid scores that are not renormalised and multiply the expert's INPUT;
* logits through the embedding table, bounded by ``logit_softcap``.

Serving layout (MI355X): the residual stream and its history over depth, norms and input convolutions (with their
carried rows), positions and angles, softmax, sinks, step sizes, decays, recurrent states, router scores and logits are
float; matrix products run in the activation dtype (bf16 with float accumulation, or float).  A sublayer's exit
(weighted add, depth average), the next norm and its input convolution are ONE kernel over runs of tokens
(:func:`~..ops.norm.residual_dyt`).  Per mixer, every projection of its input is ONE GEMM whose column slices the
kernels read in place; the two halves of a parallel mixer write into one buffer, already scaled, so their output
projections are one GEMM over the concatenated width.  Pre-activations of step sizes and decays come out of their
products in float and are finished inside the scans.  Tokens of a step are packed back to back
(:class:`~.common.SeqBatch`), so prefill, continued prefill, decode and mixed batches are the same code.

Checkpoint: ``config.json`` (``architecture: "Vefunex"``, ``vocab``, ``width``, ``norm.eps``, ``canon.taps``,
``residual_mult``, ``logit_softcap``, ``layers`` [...]) + ``model.safetensors`` with names ``embed``,
``l<i>.norm1|norm2`` (+ ``.alpha``, ``.b``), ``l<i>.canon1|canon2``, ``l<i>.dwa``, ``l<i>.mix.*``, ``l<i>.mlp.*``,
``final.norm``; linear weights ``[out, in]``.
"""
from __future__ import annotations

import copy
import dataclasses
import json
import math
import os

import torch
import torch.nn as nn

from ..ops import conv as C
from ..ops.attention import biased_attention, rope_kv_store, rotary_inv_freq
from ..ops.conv import short_conv
from ..ops.embedding import embed_pair
from ..ops.gemm import matmul_f32
from ..ops.moe import moe_glu_experts, route_tokens
from ..ops.norm import head_norm_gate, residual_dyt
from ..ops.recurrent import gated_linear_scan, selective_scan
from .common import SeqBatch, SeqStateCausalLM, SeqStateModel, _HeadWeight
from .dogudra import FEW_PAIRS, _Sublayer, _act, _chunk, _f32

MIXERS = ("attention", "parallel", "gla")


@dataclasses.dataclass
class VefunexConfig:
    vocab: int
    width: int
    layers: list
    norm_eps: float = 1e-6
    taps: int = 0                            # the input convolutions' taps (0: none); the tensors decide in the end
    residual_mult: float = 1.0
    logit_softcap: float = 0.0               # 0: unbounded logits
    max_position_embeddings: int = 4096      # engine default only
    model_type: str = "vefunex"
    eos_token_id: int | None = None

    @classmethod
    def from_dict(cls, d: dict) -> "VefunexConfig":
        layers = copy.deepcopy(d["layers"])
        for lc in layers:
            if lc["type"] not in MIXERS:
                raise ValueError(f"Vefunex: unknown layer type {lc['type']!r}")
            mlp = lc.get("mlp")
            if mlp is not None:
                if mlp.get("kind", "moe") != "moe":
                    raise ValueError(f"Vefunex: unknown feed-forward kind {mlp.get('kind')!r}")
                if not 1 <= int(mlp["router"]["top"]) <= int(mlp["router"]["experts"]):
                    raise ValueError("Vefunex: router.top must be between 1 and router.experts")
            if lc["type"] == "gla":
                continue
            at = lc["mixer"]["left"] if lc["type"] == "parallel" else lc["mixer"]
            if int(at["heads"]) % int(at.get("kv_heads", at["heads"])):
                raise ValueError("Vefunex: heads must be a multiple of kv_heads")
            dims = int((at.get("rot") or {}).get("dims", 0))
            if dims % 2 or dims > int(at["dim"]):
                raise ValueError(f"Vefunex: rot.dims = {dims} must be even and at most dim")
            qt = at.get("q_temp")
            if qt and (int(qt["every"]) != qt["every"] or int(qt["every"]) < 1):
                raise ValueError("Vefunex: q_temp.every must be a positive whole number of positions")
        return cls(vocab=int(d["vocab"]), width=int(d["width"]), layers=layers,
                   norm_eps=float(d.get("norm", {}).get("eps", 1e-6)), taps=int((d.get("canon") or {}).get("taps", 0)),
                   residual_mult=float(d.get("residual_mult", 1.0)), logit_softcap=float(d.get("logit_softcap") or 0.0),
                   max_position_embeddings=int(d.get("max_position_embeddings", 4096)))

    @classmethod
    def from_pretrained(cls, path: str) -> "VefunexConfig":
        with open(os.path.join(path, "config.json")) as f:
            return cls.from_dict(json.load(f))

    def to_dict(self) -> dict:
        d = {"architecture": "Vefunex", "vocab": self.vocab, "width": self.width, "layers": self.layers,
             "norm": {"eps": self.norm_eps}, "residual_mult": self.residual_mult, "logit_softcap": self.logit_softcap}
        if self.taps:
            d["canon"] = {"taps": self.taps}
        return d

    # names the serving engine and the CLI read from any causal-LM config
    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width


def tensor_shapes(cfg: VefunexConfig, decay_rank: int = 16) -> dict[str, tuple]:
    """Every checkpoint tensor of a config and its shape.  The low rank of the gla decays is a tensor's shape, not a
    config entry."""
    Wd = cfg.width
    out = {"embed": (cfg.vocab, Wd)}

    def norm(name):
        out.update({name: (Wd,), name + ".b": (Wd,), name + ".alpha": ()})

    def attention(q, m, parts):
        H, dk, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
        G = int(m.get("kv_heads", H))
        out.update({q + "q": (H * dk, Wd), q + "k": (G * dk, Wd), q + "v": (G * dv, Wd), q + "o": (Wd, H * dv)})
        if "g" in parts:
            out[q + "g"] = (H * dv, Wd)
        if "sink" in parts:
            out[q + "sink"] = (H,)
    norm("final.norm")
    for i, lc in enumerate(cfg.layers):
        p, m, q = f"l{i}.", lc["mixer"], f"l{i}.mix."
        norm(p + "norm1")
        out[p + "dwa"] = (i + 2,)
        if cfg.taps:
            out[p + "canon1"] = (Wd, cfg.taps)
        if lc["type"] == "attention":
            attention(q, m, ())
        elif lc["type"] == "parallel":
            attention(q + "left.", m["left"], ("g", "sink"))
            r = m["right"]
            n, N, R, q = int(r["inner"]), int(r["state"]), int(r["dt_rank"]), q + "right."
            out.update({q + "in": (2 * n, Wd), q + "conv": (n, int(r["conv"])), q + "conv.b": (n,), q + "x": (R + 2 * N, n),
                        q + "dt": (n, R), q + "dt.b": (n,), q + "A_log": (n, N), q + "D": (n,), q + "o": (Wd, n)})
        else:
            H, dk, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
            out.update({q + "q": (H * dk, Wd), q + "k": (H * dk, Wd), q + "v": (H * dv, Wd), q + "g": (H * dv, Wd),
                        q + "a1": (decay_rank, Wd), q + "a2": (H * dk, decay_rank), q + "a2.b": (H * dk,),
                        q + "norm": (dv,), q + "o": (Wd, H * dv)})
        mlp = lc.get("mlp")
        if mlp is not None:
            norm(p + "norm2")
            if cfg.taps:
                out[p + "canon2"] = (Wd, cfg.taps)
            F_ = int(mlp["expert"]["ff"])
            out[p + "mlp.router"] = (int(mlp["router"]["experts"]), Wd)
            for e in range(int(mlp["router"]["experts"])):
                out.update({f"{p}mlp.e{e}.gate": (F_, Wd), f"{p}mlp.e{e}.up": (F_, Wd), f"{p}mlp.e{e}.down": (Wd, F_)})
    return out


def random_weights(cfg: VefunexConfig, seed: int = 0, decay_rank: int = 16) -> dict[str, torch.Tensor]:
    """Synthetic weights (benchmarks, smoke runs, tests): matrices ~ N(0, 1/in), norm weights near 1, small taps, the
    last layer's result dominating every depth average, step sizes and decays in a stable range."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, decay_rank).items():
        leaf = name.rsplit(".", 1)[-1]
        if leaf in ("canon1", "canon2"):
            t = torch.randn(shape, generator=g) * 0.2
        elif leaf == "conv":
            t = torch.randn(shape, generator=g) * 0.4
        elif leaf == "dwa":
            t = torch.cat([0.1 * torch.randn(shape[0] - 1, generator=g), torch.ones(1)])
        elif leaf == "A_log":
            t = torch.rand(shape, generator=g) * 3 - 1
        elif len(shape) == 2:
            t = torch.randn(shape, generator=g) / math.sqrt(shape[1])
            if name == "embed":
                t = t * math.sqrt(shape[1]) * 0.5
        elif name.endswith("dt.b"):
            t = torch.rand(shape, generator=g) * 3 - 4
        elif name.endswith("a2.b"):
            t = torch.randn(shape, generator=g) + 2
        elif leaf == "alpha":
            t = 0.5 + 0.1 * torch.rand(shape, generator=g)
        elif leaf == "sink":
            t = torch.randn(shape, generator=g)
        elif leaf == "b":
            t = 0.1 * torch.randn(shape, generator=g)
        else:                                   # norm weights, the skip of the state space
            t = 1 + 0.1 * torch.randn(shape, generator=g)
        out[name] = t.to(torch.bfloat16)
    return out


def _splits(cache, per: int = 64) -> int:
    """Key splits of a decode step: one per ``per`` cache positions, at most 32.  Fixed per cache, so a captured decode
    step keeps its launch shapes."""
    return max(1, min(32, (cache.max_len + per - 1) // per))


class TemperedAttentionMixer(_Sublayer):
    """Unrotated grouped-query attention: a query temperature that grows with the position, unit-RMS values."""

    def __init__(self, m: dict, W: dict, p: str, dtype, dev):
        super().__init__()
        self.H, self.dk, self.dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
        self.G = int(m.get("kv_heads", self.H))
        self.scale = float(m["scale"])
        qt = m.get("q_temp")
        self.temp = (float(qt["coef"]), int(qt["every"])) if qt else None
        self.nq, self.nk, self.nv = self.H * self.dk, self.G * self.dk, self.G * self.dv
        self.put("w_in", torch.cat([W[p + n].to(dtype) for n in ("q", "k", "v")], 0).to(dev).contiguous())
        self.put("w_o", _act(W[p + "o"], dtype, dev))
        self.put("inv_freq", torch.zeros(0, device=dev))

    def state_spec(self) -> dict:
        return {"k": ((self.nk,), "kv"), "v": ((self.nv,), "kv")}

    def forward(self, h, sb: SeqBatch, st: dict, eps: float):
        q = rope_kv_store(h @ self.w_in.t(), self.nq, self.nk, self.H, self.G, self.inv_freq, 0, st["k"], st["v"], sb,
                          temp=self.temp, v_eps=eps)
        o = biased_attention(q, st["k"], st["v"], None, self.H, self.G, self.scale, sb,
                             nsplit=_splits(sb.cache) if sb.decode else 1)
        return o @ self.w_o.t()


class ParallelAttentionScanMixer(_Sublayer):
    """Capped, sinked and gated attention beside a selective state space: one input GEMM, one output GEMM."""

    def __init__(self, m: dict, W: dict, p: str, dtype, dev):
        super().__init__()
        le, ri = m["left"], m["right"]
        self.ls, self.rs = float(m.get("left_scale", 1.0)), float(m.get("right_scale", 1.0))
        self.H, self.dk, self.dv = int(le["heads"]), int(le["dim"]), int(le["vdim"])
        self.G = int(le.get("kv_heads", self.H))
        self.scale, self.cap = float(le["scale"]), float(le.get("softcap") or 0.0)
        rot = le.get("rot") or {}
        self.rot_dims = int(rot.get("dims", 0))
        self.put("inv_freq", rotary_inv_freq(self.rot_dims, float(rot.get("base", 10000.0))).to(dev))
        self.nq, self.nk, self.nv, self.no = self.H * self.dk, self.G * self.dk, self.G * self.dv, self.H * self.dv
        self.put("sinks", _f32(W[p + "left.sink"], dev) if p + "left.sink" in W else None)
        self.n, self.N, self.R = int(ri["inner"]), int(ri["state"]), int(ri["dt_rank"])
        names = ("left.q", "left.k", "left.v", "left.g", "right.in")
        self.put("w_in", torch.cat([W[p + n].to(dtype) for n in names], 0).to(dev).contiguous())
        q = p + "right."
        self.put("conv_w", _f32(W[q + "conv"], dev))
        self.put("conv_b", _f32(W[q + "conv.b"], dev))
        cnt, wd = _chunk(self.n)
        self.segs = [(0, cnt, wd, C.SILU, None, 1.0)]
        self.put("w_x", _act(W[q + "x"], dtype, dev))                 # [dt | B | C]
        self.put("w_dt", _act(W[q + "dt"], dtype, dev))
        self.put("dt_bias", _f32(W[q + "dt.b"], dev))
        self.put("a_log", _f32(W[q + "A_log"], dev))
        self.put("d_skip", _f32(W[q + "D"], dev))
        self.put("w_o", torch.cat([W[p + "left.o"].to(dtype), W[q + "o"].to(dtype)], 1).to(dev).contiguous())

    def state_spec(self) -> dict:
        spec = {"k": ((self.nk,), "kv"), "v": ((self.nv,), "kv"), "S": ((self.n, self.N), "f32")}
        if self.conv_w.shape[1] > 1:
            spec["conv"] = ((self.conv_w.shape[1] - 1, self.n), "act")
        return spec

    def forward(self, h, sb: SeqBatch, st: dict, eps: float):
        T, n, N, R = h.shape[0], self.n, self.N, self.R
        P = h @ self.w_in.t()                                         # [q | k | v | gate | x | z]
        a = self.nq + self.nk + self.nv
        both = torch.empty(T, self.no + n, dtype=h.dtype, device=h.device)
        q = rope_kv_store(P[:, :a], self.nq, self.nk, self.H, self.G, self.inv_freq, self.rot_dims, st["k"], st["v"], sb,
                          half=False)
        biased_attention(q, st["k"], st["v"], None, self.H, self.G, self.scale, sb, sink=self.sinks,
                         nsplit=_splits(sb.cache) if sb.decode else 1, out=both[:, :self.no], out_scale=self.ls,
                         softcap=self.cap, gate=P[:, a:a + self.no])
        a += self.no
        x = short_conv(P[:, a:a + n], self.conv_w, st.get("conv"), self.segs, sb, eps, bias=self.conv_b)
        D = x @ self.w_x.t()
        selective_scan(x, matmul_f32(D[:, :R], self.w_dt), self.dt_bias, D[:, R:R + N], D[:, R + N:], self.a_log,
                       self.d_skip, P[:, a + n:], st["S"], sb, both[:, self.no:], self.rs)
        return both @ self.w_o.t()


class GatedLinearMixer(_Sublayer):
    def __init__(self, m: dict, W: dict, p: str, dtype, dev):
        super().__init__()
        self.H, self.dk, self.dv, self.tau = int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["tau"])
        names = ("q", "k", "v", "g", "a1")
        self.put("w_in", torch.cat([W[p + n].to(dtype) for n in names], 0).to(dev).contiguous())
        self.put("w_a2", _act(W[p + "a2"], dtype, dev))
        self.put("a_bias", _f32(W[p + "a2.b"], dev))
        self.put("norm", _f32(W[p + "norm"], dev))
        self.put("w_o", _act(W[p + "o"], dtype, dev))
        self.off = [0]
        for n in names:
            self.off.append(self.off[-1] + W[p + n].shape[0])

    def state_spec(self) -> dict:
        return {"S": ((self.H, self.dv, self.dk), "f32")}

    def forward(self, h, sb: SeqBatch, st: dict, eps: float):
        P = h @ self.w_in.t()                                         # [q | k | v | gate | decay low-rank]
        q, k, v, g, low = (P[:, a:b] for a, b in zip(self.off, self.off[1:]))
        s = gated_linear_scan(q, k, v, matmul_f32(low, self.w_a2), self.a_bias, self.tau, self.dk ** -0.5, st["S"], self.H, sb)
        return head_norm_gate(s, self.norm, g, eps, act="silu") @ self.w_o.t()


class InputWeightedFF(_Sublayer):
    """SiLU-GLU experts behind plain sigmoid scores; a chosen expert reads its token times the score."""

    def __init__(self, mlp: dict, W: dict, p: str, dtype, dev):
        super().__init__()
        self.E, self.top = int(mlp["router"]["experts"]), int(mlp["router"]["top"])
        self.put("router", _f32(W[p + "router"], dev))
        self.put("w_gu", torch.stack([torch.stack([W[f"{p}e{e}.gate"], W[f"{p}e{e}.up"]]) for e in range(self.E)])
                 .to(device=dev, dtype=dtype).contiguous())                                  # [E, 2, F, W]
        self.put("w_d", torch.stack([W[f"{p}e{e}.down"] for e in range(self.E)]).to(device=dev, dtype=dtype).contiguous())

    def forward(self, h, sb: SeqBatch):
        idx, w = route_tokens(h, self.router, None, self.top, score="sigmoid")
        few = sb.decode or h.shape[0] * self.top <= FEW_PAIRS
        return moe_glu_experts(h, self.w_gu, self.w_d, idx, w, 0.0, None, few, act="silu", weight_input=True)


class _Entry(_Sublayer):
    """What a sublayer reads: the Dynamic Tanh of the residual and, with taps, its input convolution."""

    def __init__(self, W: dict, norm: str, conv: str | None, dev):
        super().__init__()
        self.put("weight", _f32(W[norm], dev).reshape(-1))
        self.put("bias", _f32(W[norm + ".b"], dev).reshape(-1))
        self.alpha = float(W[norm + ".alpha"])
        self.put("conv", _f32(W[conv].t(), dev) if conv in W else None)                      # [taps, W]

    @property
    def taps(self) -> int:
        return 0 if self.conv is None else self.conv.shape[0]


class VefunexLayer(nn.Module):
    def __init__(self, cfg: VefunexConfig, i: int, W: dict, dtype, dev):
        super().__init__()
        lc, p = cfg.layers[i], f"l{i}."
        mixer = {"attention": TemperedAttentionMixer, "parallel": ParallelAttentionScanMixer, "gla": GatedLinearMixer}
        self.mix = mixer[lc["type"]](lc["mixer"], W, p + "mix.", dtype, dev)
        self.enter1 = _Entry(W, p + "norm1", p + "canon1", dev)
        self.ff = self.enter2 = None
        if lc.get("mlp") is not None:
            self.enter2 = _Entry(W, p + "norm2", p + "canon2", dev)
            self.ff = InputWeightedFF(lc["mlp"], W, p + "mlp.", dtype, dev)
        self.register_buffer("depth", _f32(W[p + "dwa"], dev).reshape(-1), persistent=False)
        if self.depth.numel() != i + 2:
            raise ValueError(f"Vefunex: layer {i} averages {i + 2} streams, its checkpoint has {self.depth.numel()} weights")

    def state_spec(self) -> dict:
        spec = dict(self.mix.state_spec())
        for name, e in (("canon1", self.enter1), ("canon2", self.enter2)):
            if e is not None and e.taps > 1:
                spec[name] = ((e.taps - 1, e.weight.numel()), "f32")
        return spec


class VefunexModel(SeqStateModel):
    def __init__(self, cfg: VefunexConfig, W: dict, dtype, dev):
        super().__init__()
        self.cfg, self.dtype = cfg, dtype
        self.embed_tokens = nn.Parameter(_act(W["embed"], dtype, dev), requires_grad=False)
        self.layers = nn.ModuleList([VefunexLayer(cfg, i, W, dtype, dev) for i in range(len(cfg.layers))])
        self.final = _Entry(W, "final.norm", None, dev)
        self.residual_tap = None          # a list: receives a copy of the float residual after every layer

    def state_specs(self) -> list[dict]:
        return [layer.state_spec() for layer in self.layers]

    def state_device(self):
        return self.embed_tokens.device

    def run(self, tokens: torch.Tensor, sb: SeqBatch) -> torch.Tensor:
        """Packed tokens ``[T]`` through all layers; returns the final-normed hidden states ``[T, width]``."""
        cfg, L, mult, eps = self.cfg, self.layers, self.cfg.residual_mult, self.cfg.norm_eps
        streams = torch.empty(len(L) + 1, tokens.numel(), cfg.width, dtype=torch.float32, device=self.embed_tokens.device)
        x, _ = embed_pair(tokens, self.embed_tokens, None, None, 1.0, 0, 0, sb, out=streams[0])

        def step(x, y, e: _Entry, layer: int, state: str, n: int = 0, depth=None):
            return residual_dyt(x, y, mult, e.weight, e.bias, e.alpha, self.dtype, e.conv,
                                sb.cache.layers[layer].get(state) if e.conv is not None else None, streams, n, depth, sb)
        x, h = step(x, None, L[0].enter1, 0, "canon1")
        for i, layer in enumerate(L):
            y = layer.mix(h, sb, sb.cache.layers[i], eps)
            if layer.ff is not None:
                x, h = step(x, y, layer.enter2, i, "canon2")
                y = layer.ff(h, sb)
            last = i + 1 == len(L)
            x, h = step(x, y, self.final if last else L[i + 1].enter1, i if last else i + 1, "canon1", i + 1, layer.depth)
            if self.residual_tap is not None:
                self.residual_tap.append(x.clone())
        return h


class VefunexForCausalLM(SeqStateCausalLM):
    """Vefunex on the shared sequence-state causal-LM frame (``models/common.py``); the head is the embedding table."""

    config_class = VefunexConfig

    def __init__(self, cfg: VefunexConfig, weights: dict[str, torch.Tensor], dtype=torch.bfloat16, device=None):
        super().__init__()
        dev = torch.device(device or "cpu")
        cfg = dataclasses.replace(cfg, taps=weights["l0.canon1"].shape[1] if "l0.canon1" in weights else 0)
        rank = next((t.shape[0] for k, t in weights.items() if k.endswith("mix.a1")), 16)
        missing = [k for k in tensor_shapes(cfg, rank) if k not in weights]
        if missing:
            raise KeyError(f"Vefunex checkpoint lacks {missing[:6]}")
        self.config = cfg
        self.model = VefunexModel(cfg, weights, dtype, dev)
        self.lm_head = _HeadWeight(self.model.embed_tokens)
        self.logit_softcap = cfg.logit_softcap
        self.eval()

    @classmethod
    def from_config(cls, cfg: VefunexConfig, dtype=torch.bfloat16, device=None, seed: int = 0, decay_rank: int = 16):
        return cls(cfg, random_weights(cfg, seed, decay_rank), dtype, device)
