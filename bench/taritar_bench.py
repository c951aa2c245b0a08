"""Prefill and decode throughput of Taritar beside the closest existing models of equal layer sizes
(bench.py --taritar): a Mixtral-type model (grouped-query attention + routed experts in every layer)
and a dense Llama. Taritar alternates dense and routed feed-forwards of those sizes, keeps four residual
streams, and its second half of layers reads the keys and values of the last layer of the first half.

All models are random-init bf16 and run through the same engine and the same measurement as
bench/dofivik_bench.py: prefill is ONE step of `prompts` x `prompt_len` tokens, decode is `decode_batch`
sequences at context `context` generating greedily (HIP-graph steps, sampling included).
"""
from __future__ import annotations

import importlib.util
import json
import os


def taritar_layers(n_layers, heads, kv, dim, window, keep, ff, experts, top, e_ff, s_ff):
    att = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "softcap": 30.0,
           "mask": {"size": window, "keep_first": keep}, "rot": {"base": 500000.0, "dims": dim}}
    dense = {"kind": "dense", "ff": ff, "limit": 7.0}
    moe = {"kind": "moe", "expert": {"ff": e_ff, "limit": 7.0}, "shared": {"ff": s_ff, "limit": 7.0},
           "router": {"experts": experts, "top": top, "groups": {"count": 4, "keep": 2}}}
    half = n_layers // 2
    return [{"type": "attention", "mixer": dict(att) if i < half else dict(att, kv_from=half - 1),
             "mlp": dict(moe if i % 2 else dense)} for i in range(n_layers)]


SIZES = {
    # name: width, layers, vocab, streams, taritar sizes, mixtral / llama (heads, kv heads, head dim, expert ff, dense ff)
    "1b-class": dict(width=2048, layers=8, vocab=32000, streams=4,
                     tar=dict(heads=32, kv=8, dim=64, window=1024, keep=4, ff=8192, experts=8, top=2, e_ff=2048, s_ff=2048),
                     ref=dict(heads=32, kv=8, hd=64, e_ff=2048, ff=8192, experts=8, top=2)),
    "8b-class": dict(width=4096, layers=4, vocab=32000, streams=4,
                     tar=dict(heads=32, kv=8, dim=128, window=4096, keep=4, ff=14336, experts=8, top=2, e_ff=3584, s_ff=3584),
                     ref=dict(heads=32, kv=8, hd=128, e_ff=3584, ff=14336, experts=8, top=2)),
}


def run(a) -> int:
    import torch
    from xgserve.models import build_model
    from xgserve.models.config import ModelConfig, taritar_config
    if not torch.cuda.is_available():
        print("bench.py --taritar needs a GPU")
        return 2
    here = os.path.dirname(os.path.abspath(__file__))
    spec = importlib.util.spec_from_file_location("dofivik_bench", os.path.join(here, "dofivik_bench.py"))
    common = importlib.util.module_from_spec(spec)
    spec.loader.exec_module(common)
    dev = torch.device("cuda", 0)
    results = []
    for name in a.taritar_sizes.split(","):
        s = SIZES[name]
        tcfg = taritar_config(f"taritar-{name}", s["width"], s["vocab"], taritar_layers(s["layers"], **s["tar"]),
                              streams=s["streams"], embed_scale=2.0, logit_softcap=30.0, max_position=16384)
        r = s["ref"]
        mcfg = ModelConfig(f"mixtral-{name}", "mixtral", s["width"], s["layers"], r["heads"], r["kv"], r["hd"], r["e_ff"],
                           s["vocab"], 16384, 1000000.0, num_experts=r["experts"], experts_per_token=r["top"])
        lcfg = ModelConfig(f"llama-{name}", "llama", s["width"], s["layers"], r["heads"], r["kv"], r["hd"], r["ff"],
                           s["vocab"], 16384, 500000.0)
        row = {"size": name, "width": s["width"], "layers": s["layers"], "streams": s["streams"],
               "prompts": a.dofivik_prompts, "prompt_len": a.prompt_len, "decode_batch": a.concurrency,
               "context": a.dofivik_context}
        for key, cfg in (("taritar", tcfg), ("mixtral", mcfg), ("llama", lcfg)):
            if a.taritar_only and key != a.taritar_only:
                continue
            model = build_model(cfg, device=dev)
            row[key] = common.measure(model, dev, a.dofivik_prompts, a.prompt_len, a.concurrency, a.dofivik_context,
                                      a.steps, a.warmup)
            del model
            torch.cuda.empty_cache()
            print(f"# {name} {key} {row[key]}", flush=True)
        results.append(row)
    print(json.dumps({"metric": "taritar_vs_mixtral_llama_tokens_per_sec", "dtype": "bf16",
                      "data": "synthetic (random-token prompts, random-init weights)", "results": results}), flush=True)
    return 0
