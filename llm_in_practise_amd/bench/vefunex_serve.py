"""Serving throughput of the Vefunex design (tempered attention, capped attention beside a selective state space, gated
linear attention; depth-averaged residual with Dynamic-Tanh norms and two input convolutions per layer; input-weighted
experts) beside Dogudra — the framework's closest design on the same sequence-state path: attention, state-space layers
and routed feed-forwards — and Qwen3, all at equal width, layer count, vocabulary and matrix parameter count (random
weights, layer sizes of real models).

Same procedure as :mod:`.hybrid_serve` (whose ``measure`` runs here): the serving engine's own step functions,
prefill of ``batch`` prompts of ``prompt`` tokens packed in one step, then ``decode_steps`` decode steps for the whole
batch, eager and through the captured hipGraphs.  ``bench.py --workload vefunex-serve`` calls :func:`run`; the default
workload of ``bench.py`` is untouched.
"""
from __future__ import annotations

import torch

from .dogudra_serve import SIZES as DOGUDRA_SIZES, dogudra_config
from .hybrid_serve import SIZES as HYBRID_SIZES, _params, measure

SIZES = {
    # eight layers: attention, parallel, attention, gla, twice; every feed-forward routed
    "w1024": dict(width=1024, heads=8, kv_heads=2, dim=128, lrot=64, inner=2048, state=16, dt_rank=64, gh=8, gk=64, gv=128,
                  experts=8, top=2, taps=4),
    "w2048": dict(width=2048, heads=16, kv_heads=4, dim=128, lrot=64, inner=4096, state=16, dt_rank=128, gh=16, gk=64,
                  gv=128, experts=8, top=2, taps=4),
}


def vefunex_config(s: dict, ff: int, vocab: int = 32000) -> dict:
    heads = {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": s["dim"], "vdim": s["dim"], "scale": s["dim"] ** -0.5}

    def att():
        return {"type": "attention", "mixer": {**heads, "q_temp": {"coef": 0.1, "every": 512}}}

    def par():
        return {"type": "parallel", "mixer": {
            "left": {**heads, "rot": {"base": 500000.0, "dims": s["lrot"]}, "softcap": 30.0},
            "right": {"inner": s["inner"], "state": s["state"], "dt_rank": s["dt_rank"], "conv": 4},
            "left_scale": 0.5, "right_scale": 0.5}}

    def gla():
        return {"type": "gla", "mixer": {"heads": s["gh"], "dim": s["gk"], "vdim": s["gv"], "tau": 16.0}}
    layers = [att(), par(), att(), gla(), att(), par(), att(), gla()]
    for lc in layers:
        lc["mlp"] = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": s["experts"], "top": s["top"]}}
    return {"architecture": "Vefunex", "vocab": vocab, "width": s["width"], "layers": layers, "norm": {"eps": 1e-6},
            "canon": {"taps": s["taps"]}, "residual_mult": 0.5, "logit_softcap": 30.0}


def build_trio(size: str, device, vocab: int = 32000):
    """(Vefunex, Dogudra, Qwen3): same width, 8 layers, same vocabulary; the experts' width of Vefunex and the
    feed-forward width of Qwen3 are chosen so that all three hold the same number of matrix parameters (within one step
    of 64 columns)."""
    from ..models.dogudra import DogudraConfig, DogudraForCausalLM
    from ..models.qwen3 import Qwen3Config, Qwen3ForCausalLM
    from ..models.vefunex import VefunexConfig, VefunexForCausalLM
    s = SIZES[size]
    dog = DogudraForCausalLM.from_config(DogudraConfig.from_dict(dogudra_config(DOGUDRA_SIZES[size], vocab)),
                                         torch.bfloat16, device)
    target, W, L = _params(dog), s["width"], 8

    def with_ff(ff):
        return VefunexForCausalLM.from_config(VefunexConfig.from_dict(vefunex_config(s, ff, vocab)), torch.bfloat16, device)
    p0 = _params(with_ff(64))
    vef = with_ff(max(64, int(64 + (target - p0) / (L * s["experts"] * 3 * W)) // 64 * 64))
    hs = HYBRID_SIZES[size]
    attn = W * hs["lh"] * hs["ld"] * 2 + W * hs["lg"] * hs["ld"] * 2
    inter = max(256, int(((target - 2 * vocab * W) / L - attn) / (3 * W)) // 64 * 64)
    qcfg = Qwen3Config(vocab_size=vocab, hidden_size=W, intermediate_size=inter, num_hidden_layers=L,
                       num_attention_heads=hs["lh"], num_key_value_heads=hs["lg"], head_dim=hs["ld"],
                       max_position_embeddings=8192)
    qwen = Qwen3ForCausalLM.from_config(qcfg, dtype=torch.bfloat16, device=device).eval()
    qwen.requires_grad_(False)
    qwen.fuse_projections()
    return vef, dog, qwen


def run(sizes=("w1024", "w2048"), batch: int = 8, prompt: int = 1024, decode_steps: int = 32, vocab: int = 32000,
        device=None, models=("vefunex", "dogudra", "qwen3"), graphs=(False, True)) -> dict:
    dev = torch.device(device or "cuda")
    out = {"metric": "vefunex_serve_tokens_per_s", "unit": "tokens/s", "dtype": "bf16", "data": "synthetic",
           "batch": batch, "prompt": prompt, "decode_steps": decode_steps, "results": []}
    for size in sizes:
        trio = dict(zip(("vefunex", "dogudra", "qwen3"), build_trio(size, dev, vocab)))
        rec = {"size": size, **{f"{k}_params_m": round(_params(m) / 1e6, 1) for k, m in trio.items()}}
        rec["vefunex_expert_ff"] = trio["vefunex"].config.layers[0]["mlp"]["expert"]["ff"]
        for name in models:
            for g in graphs:
                rec[f"{name}_{'graphs' if g else 'eager'}"] = measure(trio[name], batch, prompt, decode_steps, g, vocab)
        out["results"].append(rec)
        del trio
        torch.cuda.empty_cache()
    return out
