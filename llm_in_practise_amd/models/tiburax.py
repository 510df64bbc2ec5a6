"""Tiburax: a decoder whose sublayers read the residual itself and whose norms sit on their outputs, with windowed
attention and selective-scan mixers and routed feed-forwards.

* every sublayer: ``x <- x + norm(sublayer(x))``, an RMS norm whose weight is stored as an offset from one;
* ``attention`` mixers: grouped-query attention with half-split rotation of the first ``rot.dims`` entries of each head
  (long-context frequency scaling), q and k of unit root mean square AFTER the rotation, scores bounded by ``softcap``,
  a sliding window behind which the sequence's first ``keep_first`` tokens stay visible at their true positions, and in
  all ``v_mix`` layers but the first a blend of the layer's values with the first such layer's values of the same token;
* ``mamba1`` mixers: a selective state space (short convolution + SiLU, step size per channel, decay per channel and
  state, SiLU gate);
* feed-forwards: SiLU-GLU experts, the ``top`` largest of the biased router logits weighted by the softmax over those,
  plus a shared expert for every token.

Serving layout (MI355X): the residual stream, norms, positions and angles, softmax, router, step sizes, decays and the
recurrent state are float; matrix products run in the activation dtype (bf16 with float accumulation, or float).  Per
mixer, every projection of its input is ONE GEMM whose column slices the kernels read in place.  Rotation, the heads'
norms, the value blend and the cache writes are one kernel; a sublayer's exit (norm of its output, residual sum, the next
sublayer's input in the activation dtype; after the last layer the model's norm) is one kernel.  The attention sweeps read
the kept tokens' rows and the window's rows of the cache and nothing between.  Values are cached blended; the blend reads
the first mixing layer's cached values.  Tokens of a step are packed back to back (:class:`~.common.SeqBatch`), so
prefill, continued prefill, decode and mixed batches are the same code.

Checkpoint: ``config.json`` (``architecture: "Tiburax"``, ``vocab``, ``width``, ``norm.eps``, ``embedding.scale``,
``layers`` [...]) + ``model.safetensors`` with names ``embed``, ``l<i>.norm1|norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``,
``final.norm``, ``head``; linear weights ``[out, in]``.
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
from ..ops.activation import silu_glu
from ..ops.attention import biased_attention, rope_kv_store, rotary_table
from ..ops.conv import short_conv
from ..ops.embedding import embed_pair
from ..ops.gemm import matmul_f32
from ..ops.moe import moe_glu_experts, route_tokens
from ..ops.norm import residual_postnorm
from ..ops.recurrent import selective_scan
from .common import SeqBatch, SeqStateCausalLM, SeqStateModel, _HeadWeight
from .dogudra import FEW_PAIRS, _Sublayer, _act, _chunk, _f32
from .mamivik import _window_splits

MIXERS = ("attention", "mamba1")


@dataclasses.dataclass
class TiburaxConfig:
    vocab: int
    width: int
    layers: list
    norm_eps: float = 1e-6
    embedding_scale: float = 1.0
    max_position_embeddings: int = 4096      # engine default only
    model_type: str = "tiburax"
    eos_token_id: int | None = None

    @classmethod
    def from_dict(cls, d: dict) -> "TiburaxConfig":
        layers = copy.deepcopy(d["layers"])
        first_v = None
        for i, lc in enumerate(layers):
            if lc["type"] not in MIXERS:
                raise ValueError(f"Tiburax: unknown layer type {lc['type']!r}")
            mlp = lc.get("mlp")
            if mlp is not None:
                if mlp.get("kind", "moe") != "moe":
                    raise ValueError(f"Tiburax: unknown feed-forward kind {mlp.get('kind')!r}")
                if not 1 <= int(mlp["router"]["top"]) <= int(mlp["router"]["experts"]):
                    raise ValueError("Tiburax: router.top must be between 1 and router.experts")
            if lc["type"] != "attention":
                continue
            m = lc["mixer"]
            G = int(m.get("kv_heads", m["heads"]))
            if int(m["heads"]) % G:
                raise ValueError("Tiburax: heads must be a multiple of kv_heads")
            dims = int((m.get("rot") or {}).get("dims", 0))
            if dims % 2 or dims > int(m["dim"]):
                raise ValueError(f"Tiburax: rot.dims = {dims} must be even and at most dim")
            mask = m.get("mask")
            if mask and (int(mask.get("size", 0)) < 1 or int(mask.get("keep_first", 0)) < 0):
                raise ValueError("Tiburax: mask.size must be positive and mask.keep_first not negative")
            if m.get("v_mix"):
                nv = G * int(m["vdim"])
                if first_v is not None and nv != first_v:
                    raise ValueError(f"Tiburax: layer {i} mixes {nv} value columns with the first mixing layer's {first_v}")
                first_v = nv
        return cls(vocab=int(d["vocab"]), width=int(d["width"]), layers=layers,
                   norm_eps=float(d.get("norm", {}).get("eps", 1e-6)),
                   embedding_scale=float((d.get("embedding") or {}).get("scale", 1.0)),
                   max_position_embeddings=int(d.get("max_position_embeddings", 4096)))

    @classmethod
    def from_pretrained(cls, path: str) -> "TiburaxConfig":
        with open(os.path.join(path, "config.json")) as f:
            return cls.from_dict(json.load(f))

    def to_dict(self) -> dict:
        return {"architecture": "Tiburax", "vocab": self.vocab, "width": self.width, "layers": self.layers,
                "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embedding_scale}}

    def value_source(self, i: int) -> int | None:
        """The layer whose values layer ``i`` blends into its own: the first ``v_mix`` layer, for every later one."""
        mixing = [j for j, lc in enumerate(self.layers) if lc["type"] == "attention" and lc["mixer"].get("v_mix")]
        return mixing[0] if i in mixing[1:] else None

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


def tensor_shapes(cfg: TiburaxConfig) -> dict[str, tuple]:
    """Every checkpoint tensor that a config needs, and its shape (the blend weight of the first mixing layer is not
    used and not listed)."""
    Wd = cfg.width
    out = {"embed": (cfg.vocab, Wd), "final.norm": (Wd,), "head": (cfg.vocab, Wd)}

    def glu(q, F_):
        out.update({q + "gate": (F_, Wd), q + "up": (F_, Wd), q + "down": (Wd, F_)})
    for i, lc in enumerate(cfg.layers):
        p, m, q = f"l{i}.", lc["mixer"], f"l{i}.mix."
        out[p + "norm1"] = (Wd,)
        if lc["type"] == "attention":
            H, dk, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
            G = int(m.get("kv_heads", H))
            out.update({q + "q": (H * dk, Wd), q + "k": (G * dk, Wd), q + "v": (G * dv, Wd), q + "o": (Wd, H * dv)})
            if cfg.value_source(i) is not None:
                out[q + "vmix"] = ()
        else:
            n, N, R = int(m["inner"]), int(m["state"]), int(m["dt_rank"])
            out.update({q + "in": (2 * n, Wd), q + "conv": (n, int(m["conv"])), q + "conv.b": (n,), q + "x": (R + 2 * N, n),
                        q + "dt": (n, R), q + "dt.b": (n,), q + "A_log": (n, N), q + "D": (n,), q + "o": (Wd, n)})
        mlp = lc.get("mlp")
        if mlp is not None:
            E = int(mlp["router"]["experts"])
            out.update({p + "norm2": (Wd,), p + "mlp.router": (E, Wd), p + "mlp.router.b": (E,)})
            for e in range(E):
                glu(f"{p}mlp.e{e}.", int(mlp["expert"]["ff"]))
            if mlp.get("shared") is not None:
                glu(p + "mlp.shared.", int(mlp["shared"]["ff"]))
    return out


def random_weights(cfg: TiburaxConfig, seed: int = 0) -> dict[str, torch.Tensor]:
    """Synthetic weights (benchmarks, smoke runs, tests): matrices ~ N(0, 1/in), norm offsets near 0, step sizes and
    decays in a stable range, blend weights near a half."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        if leaf == "conv":
            t = torch.randn(shape, generator=g) * 0.4
        elif leaf == "A_log":
            t = torch.rand(shape, generator=g) * 3 - 1
        elif len(shape) == 2:
            t = torch.randn(shape, generator=g) / math.sqrt(shape[1])
            if name == "embed":
                t = t * math.sqrt(shape[1]) * 0.5 / cfg.embedding_scale
        elif name.endswith("dt.b"):
            t = torch.rand(shape, generator=g) * 3 - 4
        elif leaf == "vmix":
            t = 0.3 + 0.4 * torch.rand(shape, generator=g)
        elif leaf == "D":
            t = 1 + 0.1 * torch.randn(shape, generator=g)
        else:                                   # norm offsets, biases of the convolution and the router
            t = 0.1 * torch.randn(shape, generator=g)
        out[name] = t.to(torch.bfloat16)
    return out


class KeptWindowAttentionMixer(_Sublayer):
    """Capped grouped-query attention over a sliding window and the sequence's first tokens; q and k normed after their
    rotation, values blended with an earlier layer's."""

    def __init__(self, m: dict, W: dict, p: str, dtype, dev, v_from: int | None):
        super().__init__()
        self.H, self.dk, self.dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
        self.G = int(m.get("kv_heads", self.H))
        self.scale, self.cap = float(m["scale"]), float(m.get("softcap") or 0.0)
        mask, rot = m.get("mask") or {}, m.get("rot") or {}
        self.window = int(mask.get("size", 0))
        self.keep = int(mask.get("keep_first", 0)) if self.window else 0
        self.rot_dims = int(rot.get("dims", 0))
        freq, self.mag = rotary_table(self.rot_dims, float(rot.get("base", 10000.0)), rot.get("scaling"))
        self.put("inv_freq", freq.to(dev))
        self.nq, self.nk, self.nv = self.H * self.dk, self.G * self.dk, self.G * self.dv
        self.v_from, self.lam = v_from, 0.0 if v_from is None else float(W[p + "vmix"])
        self.put("w_in", torch.cat([W[p + n].to(dtype) for n in ("q", "k", "v")], 0).to(dev).contiguous())
        self.put("w_o", _act(W[p + "o"], dtype, dev))

    def state_spec(self) -> dict:
        return {"k": ((self.nk,), "kv"), "v": ((self.nv,), "kv")}

    def forward(self, h, sb: SeqBatch, st: dict, eps: float):
        first = None if self.v_from is None else (sb.cache.layers[self.v_from]["v"], self.lam)
        q = rope_kv_store(h @ self.w_in.t(), self.nq, self.nk, self.H, self.G, self.inv_freq, self.rot_dims, st["k"], st["v"],
                          sb, True, self.mag, qk_eps=eps, v_first=first)
        reach = self.window and self.window + self.keep
        o = biased_attention(q, st["k"], st["v"], None, self.H, self.G, self.scale, sb, window=self.window,
                             nsplit=_window_splits(sb.cache, reach) if sb.decode else 1, softcap=self.cap,
                             keep_first=self.keep)
        return o @ self.w_o.t()


class SelectiveScanMixer(_Sublayer):
    def __init__(self, m: dict, W: dict, p: str, dtype, dev):
        super().__init__()
        self.n, self.N, self.R = int(m["inner"]), int(m["state"]), int(m["dt_rank"])
        self.put("w_in", _act(W[p + "in"], dtype, dev))               # [x | z]
        self.put("conv_w", _f32(W[p + "conv"], dev))
        self.put("conv_b", _f32(W[p + "conv.b"], dev))
        cnt, wd = _chunk(self.n)
        self.segs = [(0, cnt, wd, C.SILU, None, 1.0)]
        self.put("w_x", _act(W[p + "x"], dtype, dev))                 # [dt | B | C]
        self.put("w_dt", _act(W[p + "dt"], dtype, dev))
        self.put("dt_bias", _f32(W[p + "dt.b"], dev))
        self.put("a_log", _f32(W[p + "A_log"], dev))
        self.put("d_skip", _f32(W[p + "D"], dev))
        self.put("w_o", _act(W[p + "o"], dtype, dev))

    def state_spec(self) -> dict:
        spec = {"S": ((self.n, self.N), "f32")}
        if self.conv_w.shape[1] > 1:
            spec["conv"] = ((self.conv_w.shape[1] - 1, self.n), "act")
        return spec

    def forward(self, h, sb: SeqBatch, st: dict, eps: float):
        n, N, R = self.n, self.N, self.R
        P = h @ self.w_in.t()
        x = short_conv(P[:, :n], self.conv_w, st.get("conv"), self.segs, sb, eps, bias=self.conv_b)
        D = x @ self.w_x.t()
        y = selective_scan(x, matmul_f32(D[:, :R], self.w_dt), self.dt_bias, D[:, R:R + N], D[:, R + N:], self.a_log,
                           self.d_skip, P[:, n:], st["S"], sb)
        return y @ self.w_o.t()


class BiasRoutedFF(_Sublayer):
    """SiLU-GLU experts: the ``top`` largest biased logits, softmax over those; a shared expert for every token.  With few
    tokens (decode steps) a shared expert of the others' width is one more (token, expert) pair of weight 1."""

    def __init__(self, mlp: dict, W: dict, p: str, dtype, dev):
        super().__init__()
        self.E, self.top = int(mlp["router"]["experts"]), int(mlp["router"]["top"])
        self.put("router", _f32(W[p + "router"], dev))
        self.put("bias", _f32(W[p + "router.b"], dev))
        self.shared = mlp.get("shared") is not None
        self.pairs = self.shared and W[p + "shared.gate"].shape == W[p + "e0.gate"].shape
        names = [f"{p}e{e}." for e in range(self.E)] + ([p + "shared."] if self.pairs else [])
        self.put("w_gu", torch.stack([torch.stack([W[n + "gate"], W[n + "up"]]) for n in names])
                 .to(device=dev, dtype=dtype).contiguous())                                  # [E (+ 1), 2, F, W]
        self.put("w_d", torch.stack([W[n + "down"] for n in names]).to(device=dev, dtype=dtype).contiguous())
        if self.shared and not self.pairs:
            self.put("ws_gu", _act(torch.cat([W[p + "shared.gate"], W[p + "shared.up"]], 0), dtype, dev))
            self.put("ws_d", _act(W[p + "shared.down"], dtype, dev))

    def _shared(self, h):
        gu, d = (self.w_gu[-1].view(-1, h.shape[1]), self.w_d[-1]) if self.pairs else (self.ws_gu, self.ws_d)
        return silu_glu(h @ gu.t()) @ d.t()

    def forward(self, h, sb: SeqBatch):
        few = sb.decode or h.shape[0] * self.top <= FEW_PAIRS
        always = int(few and self.pairs)
        idx, w = route_tokens(h, self.router, None, self.top, normalize=True, bias=self.bias, always=always)
        sh = self._shared(h) if self.shared and not always else None
        E = self.E + always
        return moe_glu_experts(h, self.w_gu[:E], self.w_d[:E], idx, w, 0.0, sh, few, act="silu")


class TiburaxLayer(nn.Module):
    def __init__(self, cfg: TiburaxConfig, i: int, W: dict, dtype, dev):
        super().__init__()
        lc, p = cfg.layers[i], f"l{i}."
        if lc["type"] == "attention":
            self.mix = KeptWindowAttentionMixer(lc["mixer"], W, p + "mix.", dtype, dev, cfg.value_source(i))
        else:
            self.mix = SelectiveScanMixer(lc["mixer"], W, p + "mix.", dtype, dev)
        t = _Sublayer()
        t.put("norm1", 1.0 + _f32(W[p + "norm1"], dev))            # stored as an offset from one
        self.ff = None
        if lc.get("mlp") is not None:
            t.put("norm2", 1.0 + _f32(W[p + "norm2"], dev))
            self.ff = BiasRoutedFF(lc["mlp"], W, p + "mlp.", dtype, dev)
        self.t = t

    def state_spec(self) -> dict:
        return self.mix.state_spec()

    def forward(self, x, h, sb: SeqBatch, st: dict, eps: float, dtype, last_norm):
        """``x`` float residual (updated in place), ``h`` its copy in the activation dtype; returns the new ``h``, after
        the last layer (``last_norm`` given) the normed one."""
        y, w = self.mix(h, sb, st, eps), self.t.norm1
        if self.ff is not None:
            h = residual_postnorm(x, y, w, eps, dtype)
            y, w = self.ff(h, sb), self.t.norm2
        return residual_postnorm(x, y, w, eps, dtype, last_norm)


class TiburaxModel(SeqStateModel):
    split_keys = 64           # windows are short: decode wants a split per 64 cache positions

    def __init__(self, cfg: TiburaxConfig, W: dict, dtype, dev):
        super().__init__()
        self.cfg, self.dtype = cfg, dtype
        self.embed_tokens = nn.Parameter(_act(W["embed"], dtype, dev), requires_grad=False)
        self.layers = nn.ModuleList([TiburaxLayer(cfg, i, W, dtype, dev) for i in range(len(cfg.layers))])
        self.register_buffer("final_norm", 1.0 + _f32(W["final.norm"], dev), persistent=False)
        self.residual_tap = None          # a list: receives a copy of the float residual after every layer

    def state_specs(self) -> list[dict]:
        return [layer.state_spec() for layer in self.layers]

    def state_device(self):
        return self.embed_tokens.device

    def run(self, tokens: torch.Tensor, sb: SeqBatch) -> torch.Tensor:
        """Packed tokens ``[T]`` through all layers; returns the final-normed hidden states ``[T, width]``."""
        cfg, L = self.cfg, self.layers
        x, h = embed_pair(tokens, self.embed_tokens, None, None, cfg.embedding_scale, 0, 0, sb)
        for i, layer in enumerate(L):
            h = layer(x, h, sb, sb.cache.layers[i], cfg.norm_eps, self.dtype, self.final_norm if i + 1 == len(L) else None)
            if self.residual_tap is not None:
                self.residual_tap.append(x.clone())
        return h


class TiburaxForCausalLM(SeqStateCausalLM):
    """Tiburax on the shared sequence-state causal-LM frame (``models/common.py``)."""

    config_class = TiburaxConfig

    def __init__(self, cfg: TiburaxConfig, weights: dict[str, torch.Tensor], dtype=torch.bfloat16, device=None):
        super().__init__()
        dev = torch.device(device or "cpu")
        missing = [k for k in tensor_shapes(cfg) if k not in weights]
        if missing:
            raise KeyError(f"Tiburax checkpoint lacks {missing[:6]}")
        self.config = cfg
        self.model = TiburaxModel(cfg, weights, dtype, dev)
        self.lm_head = _HeadWeight(_act(weights["head"], dtype, dev))
        self.eval()

    @classmethod
    def from_config(cls, cfg: TiburaxConfig, dtype=torch.bfloat16, device=None, seed: int = 0):
        return cls(cfg, random_weights(cfg, seed), dtype, device)
