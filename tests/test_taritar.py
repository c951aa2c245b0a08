"""Taritar on the engine against the dense fp64 oracle (tests/taritar_oracle.py).

Every test runs on the CPU (PyTorch forms of the ops, same scheduler / cache code) and, marked `gpu`, on the HIP
kernels in float32 and bfloat16. Configurations and weights are made here; the oracle shares no code with xgserve.
"""
import copy
import json
import math
import os
import random
import subprocess
import sys

import pytest
import torch

import taritar_oracle as orc
from _seq_util import F64, close, engine, rel_err, run_portions, seq_meta, tokens_of
from xgserve.engine import EngineConfig, LLMEngine, SamplingParams
from xgserve.models import build_model, get_config
from xgserve.models.config import taritar_config
from xgserve.ops import seqmix as sq

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

CASES = [pytest.param("cpu", "float32", id="cpu-f32"),
         pytest.param("cuda", "float32", id="gpu-f32", marks=pytest.mark.gpu),
         pytest.param("cuda", "bfloat16", id="gpu-bf16", marks=pytest.mark.gpu)]
OP_CASES = [pytest.param("cpu", id="cpu"), pytest.param("cuda", id="gpu", marks=pytest.mark.gpu)]


def config_a():
    """Three streams; three query heads per key head; key sizes unlike value sizes; windows of five tokens with three
    kept ones, of nineteen with none, and no window; bounded and unbounded scores; rotation of a part of a head, a whole
    head, and none; keys shared from the layer before and from the first layer, with other windows and bounds than the
    owner's; routed layers with groups (with and without a shared expert) and without; a layer without feed-forward."""
    a0 = {"heads": 6, "kv_heads": 2, "dim": 20, "vdim": 12, "scale": 0.31, "softcap": 4.0,
          "mask": {"size": 5, "keep_first": 3}, "rot": {"base": 300.0, "dims": 8}}
    a1 = {"heads": 3, "kv_heads": 3, "dim": 24, "vdim": 8, "scale": 0.2}
    a2 = {"heads": 4, "kv_heads": 1, "dim": 10, "vdim": 24, "scale": 0.4, "softcap": 7.5, "mask": {"size": 19},
          "rot": {"base": 100.0, "dims": 10}}
    moe = {"kind": "moe", "expert": {"ff": 24, "limit": 1.2},
           "router": {"experts": 6, "top": 3, "groups": {"count": 3, "keep": 2}}}
    return {"architecture": "Taritar", "width": 88, "vocab": 150, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.7},
            "streams": 3, "max_positions": 230, "logit_softcap": 9.0,
            "layers": [{"type": "attention", "mixer": a0, "mlp": dict(moe, shared={"ff": 40, "limit": 0.9})},
                       {"type": "attention", "mixer": a1, "mlp": None},
                       {"type": "attention", "mixer": dict(a1, kv_from=1, heads=6, softcap=3.0, mask={"size": 7, "keep_first": 11}),
                        "mlp": {"kind": "dense", "ff": 50, "limit": 0.8}},
                       {"type": "attention", "mixer": a2, "mlp": dict(moe)},
                       {"type": "attention", "mixer": dict(a0, kv_from=0, mask={"size": 12, "keep_first": 1}, softcap=None),
                        "mlp": {"kind": "moe", "expert": {"ff": 30, "limit": 2.0}, "router": {"experts": 5, "top": 2}}}]}


def config_b():
    """Values that make mechanisms trivial: one stream, one head, one expert in one group, a window of one token without
    kept ones, a rotation of two entries, an embedding factor of one, logits without a bound."""
    a = {"heads": 1, "kv_heads": 1, "dim": 32, "vdim": 32, "scale": 0.2, "softcap": 1.0, "mask": {"size": 1, "keep_first": 0},
         "rot": {"base": 10.0, "dims": 2}}
    one = {"kind": "moe", "expert": {"ff": 32, "limit": 1.0}, "shared": {"ff": 16, "limit": 1.0},
           "router": {"experts": 1, "top": 1, "groups": {"count": 1, "keep": 1}}}
    return {"architecture": "Taritar", "width": 48, "vocab": 97, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
            "streams": 1, "max_positions": 256, "logit_softcap": None,
            "layers": [{"type": "attention", "mixer": dict(a), "mlp": one},
                       {"type": "attention", "mixer": dict(a, mask=None), "mlp": {"kind": "dense", "ff": 1, "limit": 1.0}},
                       {"type": "attention", "mixer": dict(a, kv_from=0, mask={"size": 1, "keep_first": 1}), "mlp": None}]}


def config_c():
    """Sizes the matrix-core kernels take; windows longer than a key tile and shorter, more kept tokens than a key tile
    and than the window; a bound so wide that the running maximum stays; five streams."""
    att = {"heads": 8, "kv_heads": 2, "dim": 64, "vdim": 32, "scale": 0.2, "softcap": 15.0,
           "mask": {"size": 70, "keep_first": 9}, "rot": {"base": 10000.0, "dims": 32}}
    att2 = {"heads": 4, "kv_heads": 4, "dim": 32, "vdim": 16, "scale": 0.3, "softcap": 100.0,
            "mask": {"size": 9, "keep_first": 75}, "rot": {"base": 1000.0, "dims": 32}}
    moe = {"kind": "moe", "expert": {"ff": 64, "limit": 3.0}, "shared": {"ff": 96, "limit": 2.0},
           "router": {"experts": 12, "top": 2, "groups": {"count": 4, "keep": 2}}}
    return {"architecture": "Taritar", "width": 128, "vocab": 200, "norm": {"eps": 1e-5}, "embedding": {"scale": 2.3},
            "streams": 5, "max_positions": 400, "logit_softcap": 20.0,
            "layers": [{"type": "attention", "mixer": att, "mlp": dict(moe)},
                       {"type": "attention", "mixer": att2, "mlp": {"kind": "dense", "ff": 160, "limit": 1.5}},
                       {"type": "attention", "mixer": dict(att, kv_from=0, mask={"size": 16, "keep_first": 64}), "mlp": dict(moe)},
                       {"type": "attention", "mixer": dict(att2, kv_from=1, heads=8, mask=None), "mlp": None}]}


_MADE = {}


def made(name, tmp_path_factory):
    """(config, oracle weights, checkpoint dir) of a test model, written once per session."""
    if name not in _MADE:
        cfg = {"a": config_a, "b": config_b, "c": config_c}[name]()
        Wt = orc.random_weights(cfg, seed={"a": 7, "b": 11, "c": 19}[name])
        path = str(tmp_path_factory.mktemp("taritar_" + name))
        orc.write_checkpoint(path, cfg, Wt)
        _MADE[name] = (cfg, Wt, path)
    return _MADE[name]


# ---------------------------------------------------------------------------------- whole model
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_whole_prompt_matches_oracle(name, device, dtype, tmp_path_factory):
    cfg, Wt, path = made(name, tmp_path_factory)
    toks = tokens_of(cfg, 100 if name == "c" else 45, 1)
    ref = orc.forward(cfg, Wt, toks)
    eng = engine(path, device, dtype)
    got = eng.score_step([("w", toks, list(range(len(toks))))], ["w"])
    assert close(got, ref, dtype)
    assert eng.sched.num_used_blocks() == 0


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_sum_of_streams_after_every_layer(name, device, dtype, tmp_path_factory):
    cfg, Wt, path = made(name, tmp_path_factory)
    toks = tokens_of(cfg, 17, 2)
    res = []
    orc.forward(cfg, Wt, toks, res)
    m = build_model(get_config(path), device=device, dtype=getattr(torch, dtype), checkpoint=path)
    eng = LLMEngine(EngineConfig(model=path, device=device, dtype=dtype, block_size=4, num_blocks=16, max_num_seqs=2,
                                 max_model_len=64, use_graphs=False), model=m)
    m.keep_residuals = seen = []
    eng.score_step([("x", toks, [0, 16])], ["x"])
    m.keep_residuals = None
    assert len(seen) == len(res) == len(cfg["layers"])
    for got, ref in zip(seen, res):
        assert close(got, ref, dtype)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_decode_token_by_token_equals_prefill(name, device, dtype, tmp_path_factory):
    cfg, Wt, path = made(name, tmp_path_factory)
    toks = tokens_of(cfg, 40, 3)
    ref = orc.forward(cfg, Wt, toks)
    assert close(run_portions(engine(path, device, dtype), "d", toks, []), ref, dtype)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("portions", [[2, 2, 3, 2, 9, 1, 1, 5, 2], [7, 1, 13, 2], [33, 2], [1, 2, 4, 8, 16]])
def test_portions_of_any_size(portions, device, dtype, tmp_path_factory):
    cfg, Wt, path = made("a", tmp_path_factory)
    toks = tokens_of(cfg, 42, 4)
    ref = orc.forward(cfg, Wt, toks)
    assert close(run_portions(engine(path, device, dtype), "p", toks, portions), ref, dtype)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["b", "c"])
def test_long_decoding(name, device, dtype, tmp_path_factory):
    cfg, Wt, path = made(name, tmp_path_factory)   # positions up to 170: many pages, windows pass over decoded tokens
    toks = tokens_of(cfg, 170, 5)
    ref = orc.forward(cfg, Wt, toks)
    assert close(run_portions(engine(path, device, dtype, num_blocks=48), "l", toks, [9]), ref, dtype)


@pytest.mark.parametrize("device,dtype", CASES)
def test_long_portion_after_a_short_one(device, dtype, tmp_path_factory):
    cfg, Wt, path = made("c", tmp_path_factory)
    toks = tokens_of(cfg, 250, 6)
    ref = orc.forward(cfg, Wt, toks)
    eng = engine(path, device, dtype, block_size=16, num_blocks=24, max_num_batched_tokens=512, max_model_len=400)
    assert close(run_portions(eng, "s", toks, [3, 210, 2, 35]), ref, dtype)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["a", "c"])
def test_mixed_batches_reused_pages_and_slots(name, device, dtype, tmp_path_factory):
    """Unequal requests share steps (portions beside single tokens), sit steps out, end, and later ones take
    over their slots and pages: two slots and a pool that holds only the live requests."""
    cfg, Wt, path = made(name, tmp_path_factory)
    lens = {"r0": 23, "r1": 9, "r2": 31, "r3": 1, "r4": 14}
    toks = {k: tokens_of(cfg, n, 10 + i) for i, (k, n) in enumerate(lens.items())}
    ref = {k: orc.forward(cfg, Wt, v) for k, v in toks.items()}
    eng = engine(path, device, dtype, num_blocks=14, max_num_seqs=2)
    steps = [[("r0", 5), ("r1", 2)], [("r0", 1), ("r1", 3)], [("r1", 4)], [("r0", 9)], [("r2", 6), ("r0", 1)],
             [("r0", 7), ("r2", 1)], [("r2", 2)], [("r3", 1), ("r2", 13)], [("r4", 3), ("r2", 1)], [("r2", 8), ("r4", 1)],
             [("r4", 10)]]
    at = {k: 0 for k in lens}
    got = {k: [] for k in lens}
    for st in steps:
        entries, end = [], []
        for k, n in st:
            entries.append((k, toks[k][at[k]:at[k] + n], list(range(n))))
            at[k] += n
            if at[k] == lens[k]:
                end.append(k)
        lg = eng.score_step(entries, end)
        o = 0
        for k, n in st:
            got[k].append(lg[o:o + n])
            o += n
    assert at == lens
    for k in lens:
        assert close(torch.cat(got[k], 0), ref[k], dtype), k
    assert eng.sched.num_used_blocks() == 0 and eng.sched.num_running() == 0


@pytest.mark.parametrize("device,dtype", CASES)
def test_batch_rows_equal_alone(device, dtype, tmp_path_factory):
    cfg, Wt, path = made("a", tmp_path_factory)
    a, b, c = tokens_of(cfg, 30, 20), tokens_of(cfg, 5, 21), tokens_of(cfg, 12, 22)
    eng = engine(path, device, dtype)
    alone = [eng.score_step([(n, t, list(range(len(t))))], [n]) for n, t in (("a", a), ("b", b), ("c", c))]
    both = eng.score_step([("a", a, list(range(30))), ("b", b, list(range(5))), ("c", c, list(range(12)))], ["a", "b", "c"])
    tol = 1e-5 if dtype == "float32" else 2e-2
    assert rel_err(both[:30], alone[0].cpu()) < tol and rel_err(both[30:35], alone[1].cpu()) < tol
    assert rel_err(both[35:], alone[2].cpu()) < tol


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["a", "c"])
def test_greedy_generation_through_the_scheduler(name, device, dtype, tmp_path_factory):
    """add_request / step with the engine's own scheduler (chunked prompts, several requests at once; HIP graphs
    on the GPU): every generated token is the oracle's argmax on the same history, up to rounding."""
    cfg, Wt, path = made(name, tmp_path_factory)
    prompts = [tokens_of(cfg, n, 30 + i) for i, n in enumerate((19, 3, 11, 1))]
    eng = engine(path, device, dtype, max_num_batched_tokens=8, max_num_seqs=3, use_graphs=True,
                 graph_batch_sizes=[1, 2, 4])
    outs = eng.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0, ignore_eos=True))
    assert [len(o) for o in outs] == [12] * 4
    bad = 0
    for p, o in zip(prompts, outs):
        ref = orc.forward(cfg, Wt, p + o[:-1])
        for i, tok in enumerate(o):
            row = ref[len(p) - 1 + i]
            gap = float(row.max() - row[tok])
            bad += gap > (1e-3 if dtype == "float32" else 0.15) * float(row.std())
    assert bad <= (0 if dtype == "float32" else 2)     # bfloat16: a router's close call may tip at a token


@pytest.mark.parametrize("device,dtype", CASES[:2])
def test_shared_prefix_pages_are_reused(device, dtype, tmp_path_factory):
    """Everything a sequence carries is in its pages, so a second prompt with the same beginning skips it."""
    cfg, Wt, path = made("a", tmp_path_factory)
    head = tokens_of(cfg, 24, 50)
    p1, p2 = head + tokens_of(cfg, 5, 51), head + tokens_of(cfg, 7, 52)
    sp = SamplingParams(max_tokens=8, temperature=0.0, ignore_eos=True)
    ref = [engine(path, device, dtype, enable_prefix_cache=False).generate([p], sp)[0] for p in (p1, p2)]
    eng = engine(path, device, dtype, enable_prefix_cache=True)
    assert eng.generate([p1], sp)[0] == ref[0]
    before = eng.stats_counters["prefill_tokens_computed"]
    assert eng.generate([p2], sp)[0] == ref[1]
    assert eng.stats_counters["prefill_tokens_computed"] - before <= len(p2) - 20


@pytest.mark.parametrize("device,dtype", CASES[:2])
def test_speculative_drafts_do_not_change_greedy_output(device, dtype):
    prompts = [[1, 2, 3, 4, 5], [7, 9, 11]]
    sp = SamplingParams(max_tokens=10, temperature=0.0, ignore_eos=True)
    kw = dict(model="taritar-tiny", device=device, dtype=dtype, block_size=4, num_blocks=48, max_num_seqs=2,
              max_model_len=64, use_graphs=False)
    ref = LLMEngine(EngineConfig(**kw)).generate(prompts, sp)
    out = LLMEngine(EngineConfig(draft_model="taritar-tiny", num_speculative_tokens=3, **kw)).generate(prompts, sp)
    assert out == ref


def test_registered_tiny_model_generates():
    eng = LLMEngine(EngineConfig(model="taritar-tiny", device="cpu", dtype="float32", block_size=4, num_blocks=32,
                                 max_num_seqs=2, max_model_len=64, use_graphs=False))
    outs = eng.generate([[1, 2, 3, 4, 5], [7]], SamplingParams(max_tokens=6, temperature=0.0, ignore_eos=True))
    assert [len(o) for o in outs] == [6, 6]


def test_trace_runner_cli(tmp_path, tmp_path_factory):
    cfg, Wt, path = made("b", tmp_path_factory)
    a, b = tokens_of(cfg, 21, 40), tokens_of(cfg, 6, 41)
    lines = [{"step": 0, "entries": [{"id": "a", "tokens": a[:10], "want": [0, 9]}, {"id": "b", "tokens": b[:2], "want": []}],
              "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[2:], "want": [3]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[10:], "want": [10]}], "end": ["a"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", path, "--dtype", "float32",
                        "--out", str(tmp_path / "o"), "--max-tokens", "64", "--device", "cpu"],
                       input="\n".join(json.dumps(x) for x in lines) + "\n", capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1", "done 2"]
    import numpy as np
    V = cfg["vocab"]
    ra, rb = orc.forward(cfg, Wt, a), orc.forward(cfg, Wt, b)
    g0, g1, g2 = (torch.from_numpy(np.fromfile(tmp_path / "o" / f"{i}.f32", dtype="<f4").reshape(-1, V)) for i in range(3))
    assert rel_err(g0, ra[[0, 9]]) < 2e-4 and rel_err(g1, rb[[5]]) < 2e-4 and rel_err(g2, ra[[20]]) < 2e-4


def test_save_and_reload_checkpoint(tmp_path):
    from xgserve.models import save_checkpoint
    m = build_model(get_config("taritar-tiny"), device="cpu", dtype=torch.float32, seed=3)
    save_checkpoint(m, str(tmp_path / "ck"))
    cfg2 = get_config(str(tmp_path / "ck"))
    for k in ("streams", "logit_softcap", "embed_scale", "max_position", "norm_eps", "layer_specs"):
        assert getattr(cfg2, k) == getattr(m.cfg, k), k
    m2 = build_model(cfg2, device="cpu", dtype=torch.float32, checkpoint=str(tmp_path / "ck"))
    for (n1, p1), (n2, p2) in zip(m.named_parameters(), m2.named_parameters()):
        assert n1 == n2 and torch.equal(p1.to(torch.bfloat16).float(), p2), n1
    assert m.cfg.num_params() == sum(p.numel() for p in m.parameters())
    owners = [L.mix for L in m.layers if L.mix.kv_from is None]
    assert m.cfg.kv_bytes_per_token(dtype_bytes=4) * 16 == m.cache_bytes_per_block(16) == \
        16 * 4 * sum(a.nk + a.nv for a in owners)
    cache = m.alloc_cache(4, 16, 2)
    assert cache.nbytes() == 4 * m.cache_bytes_per_block(16)       # shared pages are counted (and held) once


def test_config_rejects_what_the_design_does_not_have():
    cfg = config_a()
    for edit in (lambda L: L[0].__setitem__("type", "something_else"),
                 lambda L: L[0]["mixer"].__setitem__("kv_heads", 4),           # 6 heads do not divide over 4
                 lambda L: L[3]["mixer"]["rot"].__setitem__("dims", 12),       # more than the head holds
                 lambda L: L[0]["mixer"]["rot"].__setitem__("dims", 7),
                 lambda L: L[0]["mixer"]["mask"].__setitem__("size", 0),
                 lambda L: L[0]["mixer"]["mask"].__setitem__("keep_first", -1),
                 lambda L: L[0]["mixer"].__setitem__("softcap", -2.0),
                 lambda L: L[2]["mixer"].__setitem__("kv_from", 2),            # itself
                 lambda L: L[4]["mixer"].__setitem__("kv_from", 2),            # a layer without keys of its own
                 lambda L: L[2]["mixer"].__setitem__("kv_from", 3),            # a later layer
                 lambda L: L[4]["mixer"].__setitem__("kv_from", 1),            # other sizes
                 lambda L: L[4]["mixer"].__setitem__("rot", {"base": 301.0, "dims": 8}),
                 lambda L: L[0]["mlp"]["router"].__setitem__("top", 5),        # two groups of two experts hold four
                 lambda L: L[0]["mlp"]["router"]["groups"].__setitem__("count", 4),
                 lambda L: L[2]["mlp"].__setitem__("kind", "other")):
        bad = copy.deepcopy(cfg["layers"])
        edit(bad)
        with pytest.raises(ValueError):
            taritar_config("x", 88, 150, bad, streams=3)
    with pytest.raises(ValueError):
        taritar_config("x", 88, 150, cfg["layers"], streams=0)
    with pytest.raises(ValueError):
        taritar_config("x", 88, 150, [], streams=2)


# ---------------------------------------------------------------------------------- mechanisms alone
@pytest.mark.parametrize("device", OP_CASES)
@pytest.mark.parametrize("S", [1, 2, 3, 4, 5, 8, 11])
@pytest.mark.parametrize("T,W", [(9, 77), (5, 96), (3, 2304), (1030, 36)])
def test_residual_streams(device, S, T, W):
    """Read of equal streams, then writes with an activation branch (gated and not, strided), an fp32 term and routed rows,
    each followed by the next weighted read and its norm; the sum of the streams at the end."""
    g = torch.Generator().manual_seed(100 * S + W)
    eps = 1e-5
    rnd = lambda *s: torch.randn(*s, generator=g).to(F64)  # noqa: E731
    f = lambda t: t.float().to(device)  # noqa: E731
    x, nw = rnd(T, W), rnd(W) * 0.3 + 1.0
    w_in, w_out, mix = rnd(S), rnd(S), rnd(S, S)

    def check(X, n32, nact, ref_X, read):
        u = orc.streams_read(ref_X, read)
        ref = orc.rms_norm(u, nw, eps)
        assert float((n32.cpu().to(F64) - ref).abs().max()) < 1e-4
        assert float((nact.cpu().to(F64) - ref).abs().max()) < (1e-4 if nact.dtype == torch.float32 else 0.06)
        if X.dim() == 3:
            assert float((X.cpu().to(F64) - ref_X.transpose(0, 1)).abs().max()) < 1e-4 * float(ref_X.abs().max())
    ref_X = torch.stack([x] * S)
    X, n32, n = sq.hyper_residual(f(x), S, None, None, None, None, f(w_in), f(nw), eps, torch.float32, True)
    assert X.shape == (T, W)
    check(X, n32, n, ref_X, w_in)
    # the first write spreads the equal streams
    y = rnd(T, W + 8)
    X, n32, n = sq.hyper_residual(X, S, f(y)[:, 4:4 + W], None, f(w_out), f(mix), f(w_in), f(nw), eps, torch.bfloat16, True)
    ref_X = orc.streams_write(ref_X, mix, w_out, y[:, 4:4 + W])
    assert X.shape == (T, S, W)
    check(X, n32, n, ref_X, w_in)
    # gate per token, bfloat16 branch, fp32 term
    yb, gate, y3 = rnd(T, W).to(torch.bfloat16), torch.sigmoid(rnd(T)), rnd(T, W)
    ref_X = orc.streams_write(ref_X, mix / S, w_out, yb.to(F64) * gate[:, None] + y3)
    X, n32, n = sq.hyper_residual(X, S, yb.to(device), f(y3), f(w_out), f(mix / S), f(w_in), f(nw), eps, torch.float32, True,
                                  y_gate=f(gate))
    check(X, n32, n, ref_X, w_in)
    # routed rows in their sorted layout, two choices per token with weights; the streams are not kept
    rows, wts = rnd(2 * T + 3, W), rnd(T, 2)
    dest = torch.randperm(2 * T + 3, generator=g)[:2 * T].view(T, 2).to(torch.int32)
    y = (rows[dest.long()] * wts[:, :, None]).sum(1)
    routed = sq.RoutedRows(f(rows), dest.to(device), f(wts))
    ref_Y = orc.streams_write(ref_X, mix, w_out, y)
    before = X.clone()
    X2, n32, n = sq.hyper_residual(X, S, None, routed, f(w_out), f(mix), None, f(nw), eps, torch.float32, True, store=False)
    assert X2 is X and torch.equal(X, before)
    check(torch.empty(0), n32, n, ref_Y, torch.ones(S, dtype=F64))
    X, n32, n = sq.hyper_residual(X, S, None, routed, f(w_out), f(mix), None, f(nw), eps, torch.float32, True)
    check(X, n32, n, ref_Y, torch.ones(S, dtype=F64))


def _attention_case(device, dtype, H, G, dk, dv, bs, T, single, mask, cap, strong=None, rot=None, scale=None):
    """Queries of one sequence over scrambled pages against the oracle. `strong` = (query, key): that score stands out.
    single: the last six tokens one by one; a mixed-step twin (another sequence's single token) rides along."""
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(H * 100 + dk + T + int(mask["size"] if mask else 0))
    rnd = lambda *s: torch.randn(*s, generator=g).to(torch.bfloat16).to(F64)  # noqa: E731
    q, k, v = rnd(T, H, dk), rnd(T, G, dk), rnd(T, G, dv)
    pos = torch.arange(T)
    m = {"scale": scale or 0.4 / dk ** 0.5, "softcap": cap, "mask": mask}
    if strong is not None:
        i, j = strong
        # every head's rotated query i lines up with the rotated key j: bounded score near 0.9 cap
        back = {"base": rot["base"], "dims": rot["dims"]} if rot else None
        qi = orc.rotate(q, pos, rot)[i, ::H // G]
        k[j] = orc.rotate(qi[None], torch.tensor([-j]), back)[0] if back else qi
        for hh in range(H):
            q[i, hh] = q[i, hh // (H // G) * (H // G)]
        m["scale"] = 1.4 * cap / dk
    k, q = k.to(torch.bfloat16).to(F64), q.to(torch.bfloat16).to(F64)
    ref = orc.attend(orc.rotate(q, pos, rot), orc.rotate(k, pos, rot), v, m)
    pages = torch.randperm(80, generator=g)[:(T + bs - 1) // bs].tolist()
    kc = torch.randn(80 * bs, G * dk, generator=g).to(dt).to(device)      # stale rows everywhere
    vc = torch.randn(80 * bs, G * dv, generator=g).to(dt).to(device)
    rd = rot["dims"] if rot else 0
    table = sq.build_rot_table(rd, rot["base"], T + 1, device) if rot else None
    kind, size, keep = (sq.MASK_WINDOW, mask["size"], mask.get("keep_first", 0)) if mask else (sq.MASK_CAUSAL, 0, 0)
    out = []
    steps = [(0, T)] if not single else [(0, T - 6)] + [(T - 6 + i, 1) for i in range(6)]
    for ctx, n in steps:
        sm = seq_meta(device, [(0, ctx, n)], bs, [pages])
        src = torch.cat([q[ctx:ctx + n].reshape(n, -1), k[ctx:ctx + n].reshape(n, -1), v[ctx:ctx + n].reshape(n, -1)], 1)
        src = src.to(dt).to(device)
        qq = sq.head_norm_rope_cache(src, H, G, dk, dv, None, None, 0.0, table, rd, sm, kc, vc, dt)
        if rot:   # the queries-only form (a layer that reads another layer's keys) forms the same queries
            assert torch.equal(qq, sq.head_norm_rope_cache(src[:, :H * dk], H, 0, dk, dv, None, None, 0.0, table, rd, sm, None,
                                                           None, dt))
        out.append(sq.masked_attention(qq, kc, vc, H, G, dk, dv, kind, size, m["scale"], None, None, bs, sm,
                                       softcap=cap or 0.0, keep_first=keep))
    return torch.cat(out).float().cpu().view(T, H * dv), ref.reshape(T, H * dv)


def on(sizes, cpu):
    """(device, dtype, *sizes): every size on the GPU in both types, the first `cpu` of them on the CPU (one form serves
    all sizes there)."""
    out = []
    for i, sz in enumerate(sizes):
        name = "x".join(map(str, sz))
        if i < cpu:
            out.append(pytest.param("cpu", "float32", sz, id=f"cpu-f32-{name}"))
        for dt, tag in (("float32", "f32"), ("bfloat16", "bf16")):
            out.append(pytest.param("cuda", dt, sz, id=f"gpu-{tag}-{name}", marks=pytest.mark.gpu))
    return out


ATTN_TOL = {"float32": 1e-4, "bfloat16": 4e-2}
SHAPES = [(6, 2, 20, 12), (1, 1, 32, 32), (8, 2, 64, 32), (4, 4, 96, 48), (16, 2, 32, 128), (20, 1, 64, 64), (4, 2, 128, 128), (3, 3, 64, 128), (6, 3, 128, 64)]


@pytest.mark.parametrize("device,dtype,shape", on(SHAPES, 3))
@pytest.mark.parametrize("single", [False, True], ids=["prompt", "decoded"])
@pytest.mark.parametrize("size,keep,cap", [(7, 3, 2.0), (30, 70, 5.0), (70, 9, 80.0), (1, 1, 1.0), (64, 64, None), (0, 0, 3.0)])
def test_bounded_scores_in_windows_with_kept_tokens(device, dtype, shape, single, size, keep, cap):
    """For the general and the matrix-core kernels, as a prompt portion and as single tokens: windows and kept runs shorter
    and longer than a key tile, bounds narrow (no running maximum) and wide (with one), none, and no window at all."""
    bs = 16 if min(shape[2:]) >= 64 else 4
    got, ref = _attention_case(device, dtype, *shape, bs=bs, T=140, single=single, cap=cap,
                               mask={"size": size, "keep_first": keep} if size else None,
                               rot={"base": 50.0, "dims": shape[2] // 4 * 2})
    assert rel_err(got, ref) < ATTN_TOL[dtype]


@pytest.mark.parametrize("device,dtype,kv", on([(20, 16), (32, 16), (64, 64), (128, 128)], 1))
@pytest.mark.parametrize("size,keep", [(1, 0), (2, 5), (16, 16), (17, 1), (40, 64), (64, 4), (65, 66)])
@pytest.mark.parametrize("edge", ["window-in", "window-out", "first", "kept-in", "kept-out", "self"])
@pytest.mark.parametrize("single", [False, True], ids=["prompt", "decoded"])
def test_one_standing_out_key_at_an_edge(device, dtype, size, keep, edge, single, kv):
    """The key that stands out for the last query is the oldest one of the window or the one before it, the first / last
    kept one or the one after it, or its own: a key lost, added or read from the wrong row moves the output."""
    T = 150
    j = {"window-in": T - size, "window-out": T - 1 - size, "first": 0, "kept-in": max(keep - 1, 0), "kept-out": keep,
         "self": T - 1}[edge]
    got, ref = _attention_case(device, dtype, 4, 2, *kv, bs=16, T=T, single=single, cap=12.0,
                               mask={"size": size, "keep_first": keep}, strong=(T - 1, j), rot={"base": 500.0, "dims": 16})
    assert rel_err(got[-1:], ref[-1:]) < ATTN_TOL[dtype]
    assert rel_err(got, ref) < ATTN_TOL[dtype]


@pytest.mark.parametrize("device,dtype,kv", on([(32, 16), (64, 64)], 1))
@pytest.mark.parametrize("back", [0, 1, 15, 16, 17, 63, 64, 127, 128, 130, 299, 300])
@pytest.mark.parametrize("single", [False, True], ids=["prompt", "decoded"])
def test_far_key_without_a_window(device, dtype, back, single, kv):
    T = 301
    got, ref = _attention_case(device, dtype, 4, 2, *kv, bs=16, T=T, single=single, cap=12.0, mask=None,
                               strong=(T - 1, T - 1 - back), rot={"base": 1e4, "dims": 32})
    assert rel_err(got[-1:], ref[-1:]) < ATTN_TOL[dtype]
    assert rel_err(got, ref) < ATTN_TOL[dtype]


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("cap", [0.5, 60.0, 300.0])
def test_scores_far_beyond_the_bound(device, dtype, cap):
    """Scores hundreds of times the bound saturate: finite, and every saturated key weighs the same."""
    H, G, dk, dv, T = 2, 1, 32, 16, 70
    g = torch.Generator().manual_seed(3)
    dt = getattr(torch, dtype)
    u = torch.randn(dk, generator=g)
    sign = torch.where(torch.arange(T) % 3 == 0, 1.0, -1.0)
    k = (sign[:, None] * u[None, :]).to(dt)
    v = torch.randn(T, dv, generator=g).to(dt)
    q = torch.cat([u, -u]).repeat(T, 1).to(dt)
    kc, vc = torch.zeros(80, dk, dtype=dt, device=device), torch.zeros(80, dv, dtype=dt, device=device)
    kc[:T], vc[:T] = k.to(device), v.to(device)
    for rows in ([(0, 0, T)], [(0, T - 1, 1)]):
        sm = seq_meta(device, rows, 16, [[0, 1, 2, 3, 4]])
        o = sq.masked_attention(q[-rows[0][2]:].to(device), kc, vc, H, G, dk, dv, sq.MASK_CAUSAL, 0, 1000.0 * cap, None, None,
                                16, sm, softcap=cap).float().cpu().view(-1, H, dv)[-1]
        z = torch.stack([sign, -sign]).to(F64) * cap
        ref = torch.softmax(z, -1) @ v.to(F64)
        assert float((o.to(F64) - ref).abs().max()) < (1e-5 if dtype == "float32" else 2e-2) * float(v.abs().max())


@pytest.mark.parametrize("device,dtype", CASES[1:])
@pytest.mark.parametrize("G,dk,dv,rep", [(2, 64, 64, 4), (1, 128, 128, 8), (4, 32, 16, 1), (2, 64, 128, 16)])
def test_batches_of_single_tokens_with_unequal_contexts(device, dtype, G, dk, dv, rep):
    """A decoding step of seven sequences (contexts from one token to hundreds, a padding row) against each alone."""
    H, bs, dt = G * rep, 16, getattr(torch, dtype)
    g = torch.Generator().manual_seed(dk + rep)
    ctx = [0, 3, 15, 16, 63, 200, 331]
    tables, at = [], 0
    perm = torch.randperm(64, generator=g).tolist()
    for c in ctx:
        n = c // bs + 1
        tables.append(perm[at:at + n])
        at += n
    kc = torch.randn(64 * bs, G * dk, generator=g).to(dt).to(device)
    vc = torch.randn(64 * bs, G * dv, generator=g).to(dt).to(device)
    q = torch.randn(len(ctx), H * dk, generator=g).to(dt).to(device)
    for kind, size, keep, cap in ((sq.MASK_CAUSAL, 0, 0, 6.0), (sq.MASK_WINDOW, 50, 20, 6.0), (sq.MASK_WINDOW, 50, 20, 0.0),
                                  (sq.MASK_WINDOW, 130, 3, 99.0)):
        args = (kc, vc, H, G, dk, dv, kind, size, 0.3, None, None, bs)
        both = sq.masked_attention(q, *args, seq_meta(device, [(i, c, 1) for i, c in enumerate(ctx)], bs, tables), softcap=cap,
                                   keep_first=keep)
        m = {"scale": 0.3, "softcap": cap, "mask": {"size": size, "keep_first": keep} if size else None}
        for i, c in enumerate(ctx):
            rows = torch.tensor([tables[i][p // bs] * bs + p % bs for p in range(c + 1)])
            k, v = kc.cpu()[rows].to(F64).view(-1, G, dk), vc.cpu()[rows].to(F64).view(-1, G, dv)
            qq = torch.zeros(c + 1, H, dk, dtype=F64)
            qq[c] = q[i].cpu().to(F64).view(H, dk)
            vis = orc.visible(c, m["mask"])
            ref = torch.zeros(H, dv, dtype=F64)
            for h in range(H):
                sc = k[vis, h // rep] @ qq[c, h] * 0.3
                sc = cap * torch.tanh(sc / cap) if cap else sc
                ref[h] = torch.softmax(sc, 0) @ v[vis, h // rep]
            assert rel_err(both[i].float().cpu().view(1, -1), ref.view(1, -1)) < ATTN_TOL[dtype], (i, size, keep, cap)


@pytest.mark.parametrize("device,dtype", CASES[1:])
@pytest.mark.parametrize("G,dk,dv,rep", [(2, 64, 64, 4), (1, 128, 128, 2), (2, 64, 128, 1), (1, 32, 16, 3)])
def test_batches_of_unequal_portions(device, dtype, G, dk, dv, rep):
    """Portions of 1 to 200 tokens on contexts of 0 to 300, a sequence without a slot among them, in one launch."""
    H, bs, dt = G * rep, 16, getattr(torch, dtype)
    g = torch.Generator().manual_seed(dk + rep)
    seqs = [(0, 0, 70), (1, 300, 1), (-1, 5, 9), (2, 17, 200), (3, 250, 33), (4, 129, 2), (5, 0, 1)]
    perm = torch.randperm(96, generator=g).tolist()
    tables, at = [], 0
    for _, c, n in seqs:
        k = (c + n + bs - 1) // bs
        tables.append(perm[at:at + k])
        at += k
    kc = torch.randn(96 * bs, G * dk, generator=g).to(dt).to(device)
    vc = torch.randn(96 * bs, G * dv, generator=g).to(dt).to(device)
    q = torch.randn(sum(n for _, _, n in seqs), H * dk, generator=g).to(dt).to(device)
    for kind, size, keep, cap in ((sq.MASK_CAUSAL, 0, 0, 6.0), (sq.MASK_WINDOW, 50, 20, 6.0), (sq.MASK_WINDOW, 21, 100, 0.0),
                                  (sq.MASK_WINDOW, 130, 3, 99.0)):
        both = sq.masked_attention(q, kc, vc, H, G, dk, dv, kind, size, 0.3, None, None, bs, seq_meta(device, seqs, bs, tables),
                                   softcap=cap, keep_first=keep)
        m = {"scale": 0.3, "softcap": cap, "mask": {"size": size, "keep_first": keep} if size else None}
        o = 0
        for i, (slot, c, n) in enumerate(seqs):
            rows = torch.tensor([tables[i][p // bs] * bs + p % bs for p in range(c + n)])
            if slot >= 0:
                k, v = kc.cpu()[rows].to(F64).view(-1, G, dk), vc.cpu()[rows].to(F64).view(-1, G, dv)
                qq = torch.zeros(c + n, H, dk, dtype=F64)
                qq[c:] = q[o:o + n].cpu().to(F64).view(n, H, dk)
                ref = orc.attend(qq, k, v, m)[c:]
                assert rel_err(both[o:o + n].float().cpu(), ref.reshape(n, -1)) < ATTN_TOL[dtype], (i, size, keep, cap)
            o += n


@pytest.mark.parametrize("device", OP_CASES)
@pytest.mark.parametrize("T,E,count,keep,top", [(7, 6, 3, 2, 3), (300, 8, 2, 1, 2), (40, 1, 1, 1, 1), (33, 12, 4, 4, 5),
                                                (9, 72, 6, 2, 4), (64, 5, 1, 1, 5), (270, 16, 16, 3, 3)])
def test_router_rates_groups_by_their_best_member(device, T, E, count, keep, top):
    """Softmax scores over all experts as weights; with and without the gate's extra logit, with the logits formed by the
    kernel and given."""
    g = torch.Generator().manual_seed(E * 10 + T)
    W = 40
    rows = torch.randn(T, W, generator=g).to(F64)
    rw = torch.randn(E + 1, W, generator=g).to(F64) * 2.0 / math.sqrt(W)
    router = {"groups": {"count": count, "keep": keep}, "top": top}
    ref = [orc.route(rows[t] @ rw[:E].T, router) for t in range(T)]
    gate_ref = torch.sigmoid(rows @ rw[E])
    f = lambda t: t.float().to(device)  # noqa: E731
    for extra in (False, True):
        w = rw if extra else rw[:E]
        for kw in (dict(logits=None, rows=f(rows), router_w=f(w).contiguous()), dict(logits=f(rows @ w.T))):
            lg = kw.pop("logits")
            ids, wts, gate = sq.grouped_router(lg, None, count, keep, top, 1.0, score=sq.SCORE_SOFTMAX, rating=sq.RATE_MAX,
                                               extra_gate=extra, want_gate=True, **kw)
            for t in range(T):
                want = dict((e, float(s)) for e, s in ref[t])
                have = dict(zip(ids[t].tolist(), wts[t].tolist()))
                assert set(want) == set(have), t
                assert all(abs(want[e] - have[e]) < 1e-5 for e in want)
            assert (gate is None) == (not extra)
            if extra:
                assert float((gate.cpu().to(F64) - gate_ref).abs().max()) < 1e-5
    # a group whose two members are good together loses to one with the single best member
    lg = torch.tensor([[1.0, 1.0, 1.5, -3.0]], device=device)
    ids, _ = sq.grouped_router(lg, None, 2, 1, 1, 1.0, score=sq.SCORE_SOFTMAX, rating=sq.RATE_MAX)
    assert ids.tolist() == [[2]]
    ids, _ = sq.grouped_router(lg, None, 2, 1, 1, 1.0, score=sq.SCORE_SOFTMAX)
    assert ids.tolist()[0][0] in (0, 1)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("T,ff,limit", [(5, 50, 0.7), (9, 64, 1.0), (300, 1028, 2.5)])
def test_clamped_gate_of_dense_layers(device, dtype, T, ff, limit):
    """Gate bounded above only, up bounded on both sides and shifted by one; column counts with and without whole quads."""
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(T)
    x = (torch.randn(T, 2 * ff + 3, generator=g) * 3.0).to(dt)
    a, u = x[:, :ff].to(F64).clamp(max=limit), x[:, ff:2 * ff].to(F64).clamp(-limit, limit)
    ref = a * torch.sigmoid(1.702 * a) * (u + 1.0)
    for view in (x.to(device)[:, :2 * ff], x[:, :2 * ff].contiguous().to(device)):
        got = sq.glu_act(view, sq.GLU_CLAMPED, limit)
        assert float((got.float().cpu().to(F64) - ref).abs().max()) < \
            (1e-6 if dtype == "float32" else 2 ** -8) * float(ref.abs().max())


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("T,E,top,K,F_", [(7, 5, 2, 40, 24), (50, 1, 1, 32, 16), (100, 1, 1, 64, 32), (300, 3, 3, 64, 48),
                                          (700, 4, 1, 96, 64), (1300, 4, 2, 128, 32), (64, 12, 1, 24, 10),
                                          (900, 4, 2, 256, 128), (300, 3, 3, 256, 256), (2100, 5, 1, 512, 384)])
def test_routed_experts_with_a_clamped_gate(device, dtype, T, E, top, K, F_):
    """Every grouped-GEMM path; softmax weights at the output; the sum over choices inside the residual write."""
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(T + E)
    mlp = {"router": {"experts": E, "top": top}, "expert": {"ff": F_, "limit": 0.8}}
    w = {"router": torch.randn(E, K, generator=g).to(F64) * 3.0 / math.sqrt(K)}
    for e in range(E):
        for nm, o, i in (("gate", F_, K), ("up", F_, K), ("down", K, F_)):
            w[f"e{e}.{nm}"] = (torch.randn(o, i, generator=g) / math.sqrt(i)).to(torch.bfloat16).to(F64)
    h = torch.randn(T, K, generator=g).to(torch.bfloat16).to(F64)
    ref = orc.moe(h, w, "", mlp)
    f = lambda t: t.float().to(device)  # noqa: E731
    ids, wts = sq.grouped_router(f(h @ w["router"].T), None, 1, 1, top, 1.0, score=sq.SCORE_SOFTMAX, rating=sq.RATE_MAX)
    w13 = torch.stack([torch.cat([w[f"e{e}.gate"], w[f"e{e}.up"]]) for e in range(E)]).to(dt).to(device)
    w2 = torch.stack([w[f"e{e}.down"] for e in range(E)]).to(dt).to(device)
    got = sq.routed_experts(h.to(dt).to(device), w13, w2, ids, wts, sq.GLU_CLAMPED, 0.8)
    tol = 1e-4 if dtype == "float32" else 3e-2
    assert rel_err(got, ref) < tol
    rows = sq.routed_experts(h.to(dt).to(device), w13, w2, ids, wts, sq.GLU_CLAMPED, 0.8, combine=False)
    one = torch.ones(1, device=device)
    X, _, _ = sq.hyper_residual(torch.zeros(T, 1, K, device=device), 1, None, rows, one, torch.ones(1, 1, device=device), None,
                                torch.ones(K, device=device), 1e-5, torch.float32)
    assert rel_err(X[:, 0], ref) < tol


@pytest.mark.parametrize("device,dtype", CASES)
def test_bounded_logits(device, dtype):
    dt = getattr(torch, dtype)
    x = torch.cat([torch.linspace(-60, 60, 501), torch.tensor([1e4, -1e4, 0.0])]).to(dt).view(2, -1)
    y = sq.soft_cap_(x.clone().to(device), 7.0)
    ref = 7.0 * torch.tanh(x.to(F64) / 7.0)
    assert float((y.float().cpu().to(F64) - ref).abs().max()) < (1e-5 if dtype == "float32" else 0.02)


@pytest.mark.parametrize("device,dtype", CASES)
def test_embedding_scale_leaves_positions_unscaled(device, dtype):
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(1)
    for W in (24, 37):
        E, P = torch.randn(11, W, generator=g).to(dt), torch.randn(9, W, generator=g).to(dt)
        ids, pos = torch.tensor([3, 0, 10, 3], dtype=torch.int32), torch.tensor([8, 0, 5, 1], dtype=torch.int32)
        got = sq.embed_rows(ids.to(device), E.to(device), P.to(device), pos.to(device), 3.5)
        ref = E.to(F64)[ids.long()] * 3.5 + P.to(F64)[pos.long()]
        assert float((got.cpu().to(F64) - ref).abs().max()) < 1e-5


# ---------------------------------------------------------------------------------- random configurations
def _random_config(rng):
    def att(layers):
        own = [i for i, L in enumerate(layers) if "kv_from" not in L["mixer"]]
        mask = {"size": rng.choice([1, 3, 16, 30, 64, 100]), "keep_first": rng.choice([0, 1, 4, 20, 70])}
        mask = mask if rng.random() < 0.8 else None
        cap = rng.choice([None, 2.0, 10.0, 50.0, 120.0])
        if own and rng.random() < 0.5:
            src = rng.choice(own)
            o = layers[src]["mixer"]
            m = {k: o[k] for k in ("kv_heads", "dim", "vdim", "rot") if k in o}
            m.update(kv_from=src, heads=o["kv_heads"] * rng.choice([1, 2, 5]))
        else:
            G, dk = rng.choice([1, 2, 3]), rng.choice([16, 24, 32, 64])
            m = {"heads": G * rng.choice([1, 2, 4]), "kv_heads": G, "dim": dk, "vdim": rng.choice([8, 16, 40, 64])}
            rd = rng.choice([0, 2, dk // 4 * 2, dk])
            if rd:
                m["rot"] = {"base": rng.choice([100.0, 10000.0]), "dims": rd}
        m.update(scale=round(1.5 * m["dim"] ** -0.5, 6), mask=mask)
        if cap:
            m["softcap"] = cap
        return m
    layers = []
    for _ in range(rng.choice([2, 3, 4, 5])):
        mixer = att(layers)
        kind = rng.choice(["dense", "moe", "moe", None])
        mlp = None
        if kind == "dense":
            mlp = {"kind": "dense", "ff": rng.choice([40, 64, 130]), "limit": rng.choice([0.5, 1.0, 7.0])}
        elif kind == "moe":
            count = rng.choice([1, 2, 4])
            per = rng.choice([1, 2, 3])
            keep = rng.randrange(1, count + 1)
            mlp = {"kind": "moe", "expert": {"ff": rng.choice([16, 32, 40]), "limit": rng.choice([0.5, 2.0])},
                   "router": {"experts": count * per, "top": rng.randrange(1, min(keep * per, 3) + 1),
                              "groups": {"count": count, "keep": keep}}}
            if rng.random() < 0.7:
                mlp["shared"] = {"ff": rng.choice([16, 24, 64]), "limit": rng.choice([0.5, 2.0])}
        layers.append({"type": "attention", "mixer": mixer, "mlp": mlp})
    return {"architecture": "Taritar", "width": rng.choice([64, 96, 160, 90]), "vocab": rng.choice([97, 300]),
            "norm": {"eps": rng.choice([1e-5, 1e-6])}, "embedding": {"scale": rng.choice([0.7, 1.0, 3.0])},
            "streams": rng.choice([1, 2, 3, 4, 6]), "max_positions": 256, "logit_softcap": rng.choice([None, 5.0, 30.0]),
            "layers": layers}


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("seed", [2, 71, 82, 818, 28])
def test_random_configurations_through_mixed_schedules(seed, device, dtype, tmp_path):
    rng = random.Random(seed)
    cfg = _random_config(rng)
    Wt = orc.random_weights(cfg, seed)
    orc.write_checkpoint(str(tmp_path), cfg, Wt)
    lens = [rng.choice([150, 185]), rng.randrange(2, 20), rng.randrange(20, 45), 1]
    toks = [tokens_of(cfg, n, seed + i) for i, n in enumerate(lens)]
    refs = [orc.forward(cfg, Wt, t) for t in toks]
    eng = engine(str(tmp_path), device, dtype, block_size=16, num_blocks=sum((n + 63) // 64 * 64 for n in lens) // 16,
                 max_num_seqs=4, max_model_len=256)
    at, got = [0] * 4, [[] for _ in lens]
    while any(at[i] < lens[i] for i in range(4)):
        entries, who = [], []
        for i in range(4):
            if at[i] >= lens[i] or rng.random() < 0.2:
                continue
            n = min(lens[i] - at[i], rng.choice([1, 1, 2, 3, 17, 40, 140]))
            entries.append(("r%d" % i, toks[i][at[i]:at[i] + n], list(range(n))))
            who.append((i, n))
            at[i] += n
        if not entries:
            continue
        lg = eng.score_step(entries, ["r%d" % i for i, _ in who if at[i] == lens[i]])
        o = 0
        for i, n in who:
            got[i].append(lg[o:o + n])
            o += n
    for i in range(4):
        assert close(torch.cat(got[i], 0), refs[i], dtype), (i, cfg)
    assert eng.sched.num_used_blocks() == 0
