"""Prefill and decode throughput of Bazurax beside the closest existing models of equal layer sizes
(bench.py --bazurax): Lotelix (attention, linear recurrences and routed experts on the same operators),
a Mixtral-type model and a dense Llama.

All models are random-init bf16 and run through the same engine and the same measurement as
bench/dofivik_bench.py: prefill is ONE step of `prompts` x `prompt_len` tokens, decode is `decode_batch`
sequences at context `context` generating greedily (HIP-graph steps, sampling included).
"""
from __future__ import annotations

import importlib.util
import json
import os


def bazurax_layers(n_layers, heads, dim, vdim, l_heads, l_kv, l_dim, window, r_heads, r_dim, ff, experts, top, e_ff):
    decay = [1.0 - 2.0 ** (-5 - 7 * i / max(1, heads - 1)) for i in range(heads)]
    ret = {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay, "rot": {"base": 1000000.0, "dims": dim}}
    par = {"left": {"heads": l_heads, "kv_heads": l_kv, "dim": l_dim, "vdim": l_dim, "scale": l_dim ** -0.5,
                    "mask": {"size": window}},
           "right": {"heads": r_heads, "dim": r_dim, "decay_rank": 64}, "left_scale": 1.0, "right_scale": 0.5}
    dense = {"kind": "dense", "ff": ff}
    moe = {"kind": "moe", "expert": {"ff": e_ff}, "router": {"experts": experts, "top": top}}
    kinds = [("retention", ret, dense), ("retention", ret, moe), ("parallel", par, dense), ("retention", ret, moe)]
    return [{"type": kinds[i % 4][0], "mixer": dict(kinds[i % 4][1]), "mlp": dict(kinds[i % 4][2])} for i in range(n_layers)]


SIZES = {
    # name: width, layers, vocab, bazurax sizes, mixtral / llama (heads, kv heads, head dim, expert ff, dense ff)
    "1b-class": dict(width=2048, layers=8, vocab=32000,
                     baz=dict(heads=16, dim=128, vdim=128, l_heads=16, l_kv=4, l_dim=64, window=1024, r_heads=32, r_dim=64,
                              ff=8192, experts=8, top=2, e_ff=2048),
                     ref=dict(heads=32, kv=8, hd=64, e_ff=2048, ff=8192, experts=8, top=2)),
    "8b-class": dict(width=4096, layers=4, vocab=32000,
                     baz=dict(heads=32, dim=128, vdim=128, l_heads=16, l_kv=4, l_dim=128, window=4096, r_heads=64, r_dim=64,
                              ff=14336, experts=8, top=2, e_ff=3584),
                     ref=dict(heads=32, kv=8, hd=128, e_ff=3584, ff=14336, experts=8, top=2)),
}


def _module(name):
    here = os.path.dirname(os.path.abspath(__file__))
    spec = importlib.util.spec_from_file_location(name, os.path.join(here, name + ".py"))
    mod = importlib.util.module_from_spec(spec)
    spec.loader.exec_module(mod)
    return mod


def run(a) -> int:
    import torch
    from xgserve.models import build_model
    from xgserve.models.config import ModelConfig, bazurax_config, lotelix_config
    if not torch.cuda.is_available():
        print("bench.py --bazurax needs a GPU")
        return 2
    common, lotelix = _module("dofivik_bench"), _module("lotelix_bench")
    dev = torch.device("cuda", 0)
    results = []
    for name in a.bazurax_sizes.split(","):
        s = SIZES[name]
        bcfg = bazurax_config(f"bazurax-{name}", s["width"], s["vocab"], bazurax_layers(s["layers"], **s["baz"]),
                              max_position=16384)
        t = lotelix.SIZES[name]
        xcfg = lotelix_config(f"lotelix-{name}", t["width"], t["vocab"], lotelix.lotelix_layers(t["layers"], **t["lot"]),
                              embed_scale=t["width"] ** 0.5, norm_groups=2, max_position=16384)
        r = s["ref"]
        mcfg = ModelConfig(f"mixtral-{name}", "mixtral", s["width"], s["layers"], r["heads"], r["kv"], r["hd"], r["e_ff"],
                           s["vocab"], 16384, 1000000.0, num_experts=r["experts"], experts_per_token=r["top"])
        lcfg = ModelConfig(f"llama-{name}", "llama", s["width"], s["layers"], r["heads"], r["kv"], r["hd"], r["ff"],
                           s["vocab"], 16384, 500000.0)
        row = {"size": name, "width": s["width"], "layers": s["layers"], "prompts": a.dofivik_prompts,
               "prompt_len": a.prompt_len, "decode_batch": a.concurrency, "context": a.dofivik_context}
        for key, cfg in (("bazurax", bcfg), ("lotelix", xcfg), ("mixtral", mcfg), ("llama", lcfg)):
            if a.bazurax_only and key != a.bazurax_only:
                continue
            model = build_model(cfg, device=dev)
            row[key] = common.measure(model, dev, a.dofivik_prompts, a.prompt_len, a.concurrency, a.dofivik_context,
                                      a.steps, a.warmup)
            del model
            torch.cuda.empty_cache()
            print(f"# {name} {key} {row[key]}", flush=True)
        results.append(row)
    print(json.dumps({"metric": "bazurax_vs_lotelix_mixtral_llama_tokens_per_sec", "dtype": "bf16",
                      "data": "synthetic (random-token prompts, random-init weights)", "results": results}), flush=True)
    return 0
