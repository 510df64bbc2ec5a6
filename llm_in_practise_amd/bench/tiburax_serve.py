"""Serving throughput of the Tiburax design (capped attention over a sliding window and the first tokens, with q/k norms
after the rotation and values blended across layers; selective scans; norms on the sublayers' outputs; biased routing with
a shared expert) beside Vefunex — the framework's closest design on the same sequence-state path: capped attention,
selective scans and SiLU experts — and Qwen3, all at equal width, layer count, vocabulary and matrix parameter count
(random weights, layer sizes of real models).

Same procedure as :mod:`.hybrid_serve` (whose ``measure`` runs here): the serving engine's own step functions,
prefill of ``batch`` prompts of ``prompt`` tokens packed in one step, then ``decode_steps`` decode steps for the whole
batch, eager and through the captured hipGraphs.  ``bench.py --workload tiburax-serve`` calls :func:`run`; the default
workload of ``bench.py`` is untouched.
"""
from __future__ import annotations

import torch

from .hybrid_serve import SIZES as HYBRID_SIZES, _params, measure
from .vefunex_serve import SIZES as VEFUNEX_SIZES, vefunex_config

SIZES = {
    # eight layers, attention and selective scans in turn; every feed-forward routed, with a shared expert
    "w1024": dict(width=1024, heads=8, kv_heads=2, dim=96, vdim=64, window=512, keep=8, inner=2048, state=16, dt_rank=64,
                  experts=8, top=2),
    "w2048": dict(width=2048, heads=16, kv_heads=4, dim=128, vdim=128, window=512, keep=8, inner=4096, state=16,
                  dt_rank=128, experts=8, top=2),
}


def tiburax_config(s: dict, ff: int, vocab: int = 32000) -> dict:
    def att():
        return {"type": "attention", "mixer": {
            "heads": s["heads"], "kv_heads": s["kv_heads"], "dim": s["dim"], "vdim": s["vdim"], "scale": s["dim"] ** -0.5,
            "softcap": 30.0, "v_mix": True, "mask": {"size": s["window"], "keep_first": s["keep"]},
            "rot": {"base": 500000.0, "dims": s["dim"],
                    "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}}

    def scan():
        return {"type": "mamba1", "mixer": {"inner": s["inner"], "state": s["state"], "dt_rank": s["dt_rank"], "conv": 4}}
    layers = [f() for _ in range(4) for f in (att, scan)]
    for lc in layers:
        lc["mlp"] = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": s["experts"], "top": s["top"]},
                     "shared": {"ff": ff}}
    return {"architecture": "Tiburax", "vocab": vocab, "width": s["width"], "layers": layers, "norm": {"eps": 1e-6},
            "embedding": {"scale": float(s["width"]) ** 0.5}}


def build_trio(size: str, device, vocab: int = 32000):
    """(Tiburax, Vefunex, Qwen3): same width, 8 layers, same vocabulary; the experts' width of Tiburax and the feed-forward
    width of Qwen3 are chosen so that all three hold the same number of matrix parameters (within one step of 64
    columns)."""
    from ..models.qwen3 import Qwen3Config, Qwen3ForCausalLM
    from ..models.tiburax import TiburaxConfig, TiburaxForCausalLM
    from ..models.vefunex import VefunexConfig, VefunexForCausalLM
    s = SIZES[size]
    vef = VefunexForCausalLM.from_config(VefunexConfig.from_dict(vefunex_config(VEFUNEX_SIZES[size], 640 if s["width"] <= 1024 else 576,
                                                                                vocab)), torch.bfloat16, device)
    target, W, L = _params(vef), s["width"], 8

    def with_ff(ff):
        return TiburaxForCausalLM.from_config(TiburaxConfig.from_dict(tiburax_config(s, ff, vocab)), torch.bfloat16, device)
    p0 = _params(with_ff(64))
    tib = with_ff(max(64, int(64 + (target - p0) / (L * (s["experts"] + 1) * 3 * W)) // 64 * 64))
    hs = HYBRID_SIZES[size]
    attn = W * hs["lh"] * hs["ld"] * 2 + W * hs["lg"] * hs["ld"] * 2
    inter = max(256, int(((target - 2 * vocab * W) / L - attn) / (3 * W)) // 64 * 64)
    qcfg = Qwen3Config(vocab_size=vocab, hidden_size=W, intermediate_size=inter, num_hidden_layers=L,
                       num_attention_heads=hs["lh"], num_key_value_heads=hs["lg"], head_dim=hs["ld"],
                       max_position_embeddings=8192)
    qwen = Qwen3ForCausalLM.from_config(qcfg, dtype=torch.bfloat16, device=device).eval()
    qwen.requires_grad_(False)
    qwen.fuse_projections()
    return tib, vef, qwen


def run(sizes=("w1024", "w2048"), batch: int = 8, prompt: int = 1024, decode_steps: int = 32, vocab: int = 32000,
        device=None, models=("tiburax", "vefunex", "qwen3"), graphs=(False, True)) -> dict:
    dev = torch.device(device or "cuda")
    out = {"metric": "tiburax_serve_tokens_per_s", "unit": "tokens/s", "dtype": "bf16", "data": "synthetic",
           "batch": batch, "prompt": prompt, "decode_steps": decode_steps, "results": []}
    for size in sizes:
        trio = dict(zip(("tiburax", "vefunex", "qwen3"), build_trio(size, dev, vocab)))
        rec = {"size": size, **{f"{k}_params_m": round(_params(m) / 1e6, 1) for k, m in trio.items()}}
        rec["tiburax_expert_ff"] = trio["tiburax"].config.layers[0]["mlp"]["expert"]["ff"]
        for name in models:
            for g in graphs:
                rec[f"{name}_{'graphs' if g else 'eager'}"] = measure(trio[name], batch, prompt, decode_steps, g, vocab)
        out["results"].append(rec)
        del trio
        torch.cuda.empty_cache()
    return out
