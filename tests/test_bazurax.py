"""Bazurax on the engine against the dense fp64 oracle (tests/bazurax_oracle.py).

Every test runs on the CPU (PyTorch forms of the ops, same scheduler / cache / state code) and, marked `gpu`, on the HIP
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

import bazurax_oracle as orc
from _seq_util import F64, close, engine, rel_err, row_errs, run_portions, seq_meta, tokens_of
from xgserve.engine import EngineConfig, LLMEngine, SamplingParams
from xgserve.models import build_model, get_config
from xgserve.models.config import bazurax_config
from xgserve.ops import seqmix as sq

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
CASES = [pytest.param("cpu", "float32", id="cpu-f32"),
         pytest.param("cuda", "float32", id="gpu-f32", marks=pytest.mark.gpu),
         pytest.param("cuda", "bfloat16", id="gpu-bf16", marks=pytest.mark.gpu)]
OP_CASES = [pytest.param("cpu", id="cpu"), pytest.param("cuda", id="gpu", marks=pytest.mark.gpu)]


def config_a():
    """Sizes no matrix-core kernel takes; a parallel layer first; three query heads per key head; key sizes unlike value
    sizes; a window of five tokens; rotation of part of a head and none at all; a head that forgets almost everything; a
    layer without feed-forward; two of five experts, three of three."""
    par = {"left": {"heads": 6, "kv_heads": 2, "dim": 12, "vdim": 20, "scale": 0.35, "mask": {"size": 5}},
           "right": {"heads": 3, "dim": 20, "decay_rank": 6}, "left_scale": 0.7, "right_scale": -1.3}
    r0 = {"heads": 3, "dim": 20, "vdim": 12, "decay": [0.9, 0.003, 0.99], "rot": {"base": 300.0, "dims": 8}}
    r1 = {"heads": 2, "dim": 10, "vdim": 26, "decay": [0.96875, 1.0]}
    moe = {"kind": "moe", "expert": {"ff": 24}, "router": {"experts": 5, "top": 2}}
    return {"architecture": "Bazurax", "width": 88, "vocab": 150, "norm": {"eps": 1e-5},
            "layers": [{"type": "parallel", "mixer": par, "mlp": dict(moe)},
                       {"type": "retention", "mixer": r0, "mlp": None},
                       {"type": "retention", "mixer": r1, "mlp": {"kind": "dense", "ff": 72}},
                       {"type": "parallel", "mixer": dict(par, left_scale=1.0, right_scale=0.25),
                        "mlp": {"kind": "moe", "expert": {"ff": 40}, "router": {"experts": 3, "top": 3}}}]}


def config_b():
    """Values that make mechanisms trivial: one head, one expert, a window of one token, rank one, both branch scales one,
    a rotation of two entries, a width that is no multiple of four."""
    par = {"left": {"heads": 1, "kv_heads": 1, "dim": 16, "vdim": 16, "scale": 1.0, "mask": {"size": 1}},
           "right": {"heads": 1, "dim": 16, "decay_rank": 1}, "left_scale": 1.0, "right_scale": 1.0}
    ret = {"heads": 1, "dim": 32, "vdim": 32, "decay": [0.75], "rot": {"base": 10.0, "dims": 2}}
    return {"architecture": "Bazurax", "width": 50, "vocab": 97, "norm": {"eps": 1e-6},
            "layers": [{"type": "retention", "mixer": ret, "mlp": None},
                       {"type": "parallel", "mixer": par, "mlp": {"kind": "moe", "expert": {"ff": 32},
                                                                  "router": {"experts": 1, "top": 1}}},
                       {"type": "retention", "mixer": dict(ret), "mlp": {"kind": "moe", "expert": {"ff": 16},
                                                                         "router": {"experts": 4, "top": 1}}}]}


def config_c():
    """Sizes the matrix-core kernels take, in several of their forms: value sizes below, at and above one workgroup's
    columns, whole and partial rotation, a window longer than a key tile."""
    par = {"left": {"heads": 8, "kv_heads": 2, "dim": 32, "vdim": 16, "scale": 0.2, "mask": {"size": 70}},
           "right": {"heads": 2, "dim": 32, "decay_rank": 8}, "left_scale": 0.9, "right_scale": 0.6}
    par2 = {"left": {"heads": 4, "kv_heads": 4, "dim": 64, "vdim": 64, "scale": 0.125, "mask": {"size": 33}},
            "right": {"heads": 1, "dim": 64, "decay_rank": 16}, "left_scale": -0.5, "right_scale": 1.5}
    r0 = {"heads": 2, "dim": 64, "vdim": 80, "decay": [0.97, 0.999], "rot": {"base": 10000.0, "dims": 32}}
    r1 = {"heads": 3, "dim": 32, "vdim": 16, "decay": [0.5, 0.99, 0.9995], "rot": {"base": 1e6, "dims": 32}}
    r2 = {"heads": 1, "dim": 96, "vdim": 136, "decay": [0.992]}
    moe = {"kind": "moe", "expert": {"ff": 64}, "router": {"experts": 6, "top": 2}}
    return {"architecture": "Bazurax", "width": 128, "vocab": 200, "norm": {"eps": 1e-5},
            "layers": [{"type": "retention", "mixer": r0, "mlp": dict(moe)},
                       {"type": "parallel", "mixer": par, "mlp": {"kind": "dense", "ff": 160}},
                       {"type": "retention", "mixer": r1, "mlp": None},
                       {"type": "parallel", "mixer": par2, "mlp": dict(moe)},
                       {"type": "retention", "mixer": r2, "mlp": dict(moe)}]}


_MADE = {}


def made(name, tmp_path_factory):
    """(config, oracle weights, checkpoint dir) of a test model, written once per session."""
    if name not in _MADE:
        cfg = {"a": config_a, "b": config_b, "c": config_c}[name]()
        Wt = orc.random_weights(cfg, seed={"a": 6, "b": 14, "c": 22}[name])
        path = str(tmp_path_factory.mktemp("bazurax_" + name))
        orc.write_checkpoint(path, cfg, Wt)
        _MADE[name] = (cfg, Wt, path)
    return _MADE[name]


# ---------------------------------------------------------------------------------- whole model
@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_whole_prompt_matches_oracle(name, device, dtype, tmp_path_factory):
    cfg, Wt, path = made(name, tmp_path_factory)
    toks = tokens_of(cfg, 90 if name == "c" else 45, 1)
    ref = orc.forward(cfg, Wt, toks)
    eng = engine(path, device, dtype)
    got = eng.score_step([("w", toks, list(range(len(toks))))], ["w"])
    assert close(got, ref, dtype)
    assert eng.sched.num_used_blocks() == 0


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["a", "c"])
def test_residual_after_every_layer(name, device, dtype, tmp_path_factory):
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
    tol = 1e-4 if dtype == "float32" else 8e-2
    assert len(seen) == len(res) == len(cfg["layers"])
    for got, ref in zip(seen, res):
        assert float((got.detach().to("cpu", F64) - ref).abs().max()) < tol * float(ref.abs().max())


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_decode_token_by_token_equals_prefill(name, device, dtype, tmp_path_factory):
    cfg, Wt, path = made(name, tmp_path_factory)
    toks = tokens_of(cfg, 40, 3)
    ref = orc.forward(cfg, Wt, toks)
    eng = engine(path, device, dtype)
    assert close(run_portions(eng, "d", toks, []), ref, dtype)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["a", "c"])
@pytest.mark.parametrize("portions", [[2, 2, 3, 2, 9, 1, 1, 5, 2], [7, 1, 13, 2], [33, 2], [1, 2, 4, 8, 16]])
def test_portions_of_any_size(portions, name, device, dtype, tmp_path_factory):
    cfg, Wt, path = made(name, tmp_path_factory)
    toks = tokens_of(cfg, 42, 4)
    ref = orc.forward(cfg, Wt, toks)
    eng = engine(path, device, dtype)
    assert close(run_portions(eng, "p", toks, portions), ref, dtype)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["b", "c"])
def test_long_decoding(name, device, dtype, tmp_path_factory):
    """Positions up to 170: many pages, windows pass over decoded tokens."""
    cfg, Wt, path = made(name, tmp_path_factory)
    toks = tokens_of(cfg, 170, 5)
    ref = orc.forward(cfg, Wt, toks)
    eng = engine(path, device, dtype, num_blocks=48)
    assert close(run_portions(eng, "l", toks, [9]), ref, dtype)


@pytest.mark.parametrize("device,dtype", CASES)
def test_long_portion_is_cut_into_segments(device, dtype, tmp_path_factory):
    """A portion of several hundred tokens after a short one: the recurrences run it in segments side by side that start
    from the carried state."""
    cfg, Wt, path = made("c", tmp_path_factory)
    toks = tokens_of(cfg, 333, 6)
    ref = orc.forward(cfg, Wt, toks)
    eng = engine(path, device, dtype, block_size=16, num_blocks=24, max_num_batched_tokens=512, max_model_len=400)
    assert close(run_portions(eng, "s", toks, [3, 290, 2, 37]), ref, dtype)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["a", "c"])
def test_mixed_batches_reused_pages_and_slots(name, device, dtype, tmp_path_factory):
    """Unequal requests share steps (portions beside single tokens), sit steps out, end, and later ones take over their
    slots and pages: two slots and a pool that holds only the live requests."""
    cfg, Wt, path = made(name, tmp_path_factory)
    lens = {"r0": 23, "r1": 9, "r2": 31, "r3": 1, "r4": 14}
    toks = {k: tokens_of(cfg, n, 10 + i) for i, (k, n) in enumerate(lens.items())}
    ref = {k: orc.forward(cfg, Wt, v) for k, v in toks.items()}
    eng = engine(path, device, dtype, num_blocks=14, max_num_seqs=2)
    steps = [[("r0", 5), ("r1", 2)], [("r0", 1), ("r1", 3)], [("r1", 4)], [("r0", 9)], [("r2", 6), ("r0", 1)],
             [("r0", 7), ("r2", 1)], [("r2", 2)], [("r3", 1), ("r2", 13)], [("r4", 3), ("r2", 1)], [("r2", 8), ("r4", 1)],
             [("r4", 10)]]
    at, got = {k: 0 for k in lens}, {k: [] for k in lens}
    for st in steps:
        entries, end = [], []
        for k, n in st:
            entries.append((k, toks[k][at[k]:at[k] + n], list(range(n))))
            at[k] += n
            if at[k] == lens[k]:
                end.append(k)
        lg, o = eng.score_step(entries, end), 0
        for k, n in st:
            got[k].append(lg[o:o + n])
            o += n
    assert at == lens
    for k in lens:
        assert close(torch.cat(got[k], 0), ref[k], dtype), k
    assert eng.sched.num_used_blocks() == 0 and eng.sched.num_running() == 0


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["a", "c"])
def test_batch_rows_equal_alone(name, device, dtype, tmp_path_factory):
    cfg, Wt, path = made(name, tmp_path_factory)
    lens = (50, 5, 12)
    reqs = [(n, tokens_of(cfg, m, 20 + i), list(range(m))) for i, (n, m) in enumerate(zip("abc", lens))]
    eng = engine(path, device, dtype)
    alone = [eng.score_step([r], [r[0]]).cpu() for r in reqs]
    both = eng.score_step(reqs, ["a", "b", "c"])
    o = 0
    for ref, m in zip(alone, lens):
        e = row_errs(both[o:o + m], ref)
        o += m
        if dtype == "float32":
            assert float(e.max()) < 1e-5
        else:   # a router's close call may tip at a token
            assert float(e.median()) < 2e-2 and float((e > 3e-2).double().mean()) <= 0.1


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("name", ["a", "c"])
def test_greedy_generation_through_the_scheduler(name, device, dtype, tmp_path_factory):
    """add_request / step with the engine's own scheduler (chunked prompts, several requests at once; HIP graphs on the
    GPU): every generated token is the oracle's argmax on the same history, up to rounding."""
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
    assert bad <= (0 if dtype == "float32" else 2)
    assert eng.sched.num_used_blocks() == 0


def test_registered_tiny_model_generates():
    eng = LLMEngine(EngineConfig(model="bazurax-tiny", device="cpu", dtype="float32", block_size=4, num_blocks=32,
                                 max_num_seqs=2, max_model_len=64, use_graphs=False))
    outs = eng.generate([[1, 2, 3, 4, 5], [7]], SamplingParams(max_tokens=6, temperature=0.0, ignore_eos=True))
    assert [len(o) for o in outs] == [6, 6]


def test_model_without_pages_generates(tmp_path):
    """Retention layers alone: nothing is paged, the state is all a sequence carries."""
    cfg = config_c()
    cfg["layers"] = [cfg["layers"][0], cfg["layers"][2]]
    Wt = orc.random_weights(cfg, 3)
    orc.write_checkpoint(str(tmp_path), cfg, Wt)
    eng = engine(str(tmp_path), "cpu", "float32")
    toks = tokens_of(cfg, 30, 7)
    assert close(run_portions(eng, "n", toks, [11, 1, 7]), orc.forward(cfg, Wt, toks), "float32")


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
    g = [torch.from_numpy(np.fromfile(tmp_path / "o" / f"{i}.f32", dtype="<f4").reshape(-1, V)) for i in range(3)]
    assert rel_err(g[0], ra[[0, 9]]) < 2e-4 and rel_err(g[1], rb[[5]]) < 2e-4 and rel_err(g[2], ra[[20]]) < 2e-4


def test_save_and_reload_checkpoint(tmp_path):
    from xgserve.models import save_checkpoint
    m = build_model(get_config("bazurax-tiny"), device="cpu", dtype=torch.float32, seed=3)
    save_checkpoint(m, str(tmp_path / "ck"))
    cfg2 = get_config(str(tmp_path / "ck"))
    assert cfg2.norm_eps == m.cfg.norm_eps and cfg2.tie_embeddings
    assert "decay_rank" not in cfg2.layer_specs[1]["mixer"]["right"]       # read from a tensor's shape on load
    m2 = build_model(cfg2, device="cpu", dtype=torch.float32, checkpoint=str(tmp_path / "ck"))
    for (n1, p1), (n2, p2) in zip(m.named_parameters(), m2.named_parameters()):
        assert n1 == n2 and torch.equal(p1.to(torch.bfloat16).float(), p2), n1
    assert m.cfg.num_params() == sum(p.numel() for p in m.parameters())


def test_config_rejects_what_the_design_does_not_have():
    cfg = config_a()
    for edit in (lambda L: L[0].__setitem__("type", "something_else"),
                 lambda L: L[0]["mixer"]["left"].__setitem__("kv_heads", 4),       # 6 heads do not divide over 4
                 lambda L: L[0]["mixer"]["left"]["mask"].__setitem__("size", 0),
                 lambda L: L[0]["mixer"].pop("left_scale"),
                 lambda L: L[0]["mixer"]["right"].__setitem__("dim", 300),
                 lambda L: L[1]["mixer"]["decay"].append(0.5),                     # more decays than heads
                 lambda L: L[1]["mixer"]["rot"].__setitem__("dims", 22),           # more than the head holds
                 lambda L: L[1]["mixer"]["rot"].__setitem__("dims", 7),
                 lambda L: L[2]["mlp"].__setitem__("kind", "sparse"),
                 lambda L: L[0]["mlp"]["router"].__setitem__("top", 6)):
        bad = copy.deepcopy(cfg["layers"])
        edit(bad)
        with pytest.raises(ValueError):
            bazurax_config("x", 88, 150, bad)
    with pytest.raises(ValueError):
        bazurax_config("x", 88, 150, [])
    with pytest.raises(ValueError):
        LLMEngine(EngineConfig(model="bazurax-tiny", device="cpu", num_blocks=8, max_num_seqs=2, max_model_len=32,
                               use_graphs=False, draft_model="llama-tiny-draft", num_speculative_tokens=2))


# ---------------------------------------------------------------------------------- mechanisms alone
def in_portions(device, lens, cuts, slots, fn):
    """fn(list of (sequence, first row, rows)) with the step's SeqMeta, several sequences cut into portions that share
    steps; returns each sequence's outputs in order."""
    got, at = [[] for _ in lens], [0] * len(lens)
    cuts = [list(c) for c in cuts]
    while any(cuts):
        who = []
        for i in range(len(lens)):
            if cuts[i]:
                q = cuts[i].pop(0)
                who.append((i, at[i], q))
                at[i] += q
        sm = seq_meta(device, [(slots[i], a, q) for i, a, q in who], 4, [[0] * 1024 for _ in who])
        y, o = fn(who, sm), 0
        for i, _, q in who:
            got[i].append(y[o:o + q].float().cpu())
            o += q
    assert at == list(lens)
    return [torch.cat(g).to(F64) for g in got]


def bf(t):
    return t.to(torch.bfloat16).to(F64)


@pytest.mark.parametrize("device", OP_CASES)
@pytest.mark.parametrize("W", [77, 96, 1024, 2304, 4096, 5000])
def test_layer_norm_of_the_sublayer_output(device, W):
    """Embedding rows, one branch, two scaled branches (strided activations), an fp32 sum; the copy of x and the norm of x
    that follow. A common offset of the sublayer's output, a hundred times its spread, must drop out."""
    g = torch.Generator().manual_seed(W)
    T, eps = 7, 1e-5
    rnd = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    w, nw = rnd(W) * 0.3 + 1.0, rnd(W) * 0.3 + 1.0
    f = lambda t: t.float().to(device)  # noqa: E731
    table = rnd(11, W).to(torch.bfloat16)
    ids = torch.tensor([3, 0, 10, 7, 3, 11, -1], dtype=torch.int32, device=device)   # the last two: no such row
    for dt in (torch.float32, torch.bfloat16):
        x, h = sq.layer_norm_residual(None, table.to(dt).to(device), f(w), eps, dt, ids=ids)
        ref = orc.layer_norm(table[[3, 0, 10, 7, 3]].to(F64), w.to(F64), eps)
        assert float((x[:5].cpu().to(F64) - ref).abs().max()) < 2e-5 and float(x[5:].abs().max()) == 0.0
        assert h.dtype == dt and torch.equal(h, x.to(dt))
    wide = (rnd(T, 2 * W + 8) + 100.0).to(torch.bfloat16)
    ya, yb = wide[:, :W], wide[:, W + 8:]
    x0, y3 = rnd(T, W) * 3, rnd(T, W) * 0.01 + 1.0
    for mode in ("one", "two", "fp32"):
        xs = f(x0).clone()
        wd = wide.to(device)
        if mode == "one":
            u = ya.to(F64)
            _, h = sq.layer_norm_residual(xs, wd[:, :W], f(w), eps, torch.bfloat16)
        elif mode == "two":
            u = 0.7 * ya.to(F64) - 1.3 * yb.to(F64)
            _, h = sq.layer_norm_residual(xs, wd[:, :W], f(w), eps, torch.bfloat16, y2=wd[:, W + 8:], scales=(0.7, -1.3))
        else:
            u = y3.to(F64)
            _, h = sq.layer_norm_residual(xs, sq.RoutedRows(f(y3)), f(w), eps, torch.bfloat16)
        ref = x0.to(F64) + orc.layer_norm(u, w.to(F64), eps)
        tol = 2e-3 if mode == "fp32" else 2e-4   # fp32 rounding of the offset, over the spread
        assert float((xs.cpu().to(F64) - ref).abs().max()) < tol
        assert torch.equal(h, xs.to(torch.bfloat16))
        xs = f(x0).clone()
        _, n = sq.layer_norm_residual(xs, wd[:, :W], f(w), eps, torch.float32, next_w=f(nw))
        ref = orc.layer_norm(x0.to(F64) + orc.layer_norm(ya.to(F64), w.to(F64), eps), nw.to(F64), eps)
        assert float((n.cpu().to(F64) - ref).abs().max()) < 2e-4


@pytest.mark.parametrize("device", OP_CASES)
@pytest.mark.parametrize("W", [30, 64, 1100])
def test_token_shift_over_portions_and_slots(device, W):
    """Every mix reads its own share of the previous token's row: within a portion, across portions and single tokens, and
    zeros at a sequence's start whatever the slot holds."""
    g = torch.Generator().manual_seed(W)
    lens, cuts = (29, 11, 1), [[5, 1, 1, 2, 17, 1, 2], [2, 2, 1, 1, 5], [1]]
    xs = [torch.randn(n, W, generator=g) for n in lens]
    mu = torch.rand(5, W, generator=g)
    state = torch.randn(4, W, generator=g).to(device)

    def fn(who, sm):
        x = torch.cat([xs[i][a:a + q] for i, a, q in who]).to(device)
        return sq.token_shift_mix(x, mu.to(device), state, sm, torch.float32).transpose(0, 1).reshape(x.shape[0], -1)
    got = in_portions(device, lens, cuts, [2, 0, 3], fn)
    for x, y in zip(xs, got):
        ref = torch.stack([orc.token_shift(x.to(F64), mu[j].to(F64)) for j in range(5)], 1).reshape(x.shape[0], -1)
        assert float((y - ref).abs().max()) < 1e-5
    assert torch.equal(state[2].cpu(), xs[0][-1]) and torch.equal(state[0].cpu(), xs[1][-1])


RET_SHAPES = [(3, 20, 12, 8), (2, 10, 26, 0), (1, 6, 70, 2), (3, 32, 16, 32), (2, 64, 80, 32), (2, 64, 64, 64), (1, 96, 136, 0),
              (2, 128, 128, 128), (1, 128, 48, 64), (1, 256, 264, 256)]
CUTS = {"short": ((29, 11), [[5, 1, 1, 2, 17, 1, 2], [2, 2, 1, 1, 5]]),
        "single": ((9, 4), [[1] * 9, [1] * 4]),
        "long": ((420, 40), [[3, 300, 1, 77, 39], [20, 1, 2, 1, 16]])}


def _retention_case(device, dtype, H, dk, dv, rd, lens, cuts, decay, seed, tweak=None):
    """sq.retention over portions on stale slots against the oracle; (worst output error, worst state error)."""
    g = torch.Generator().manual_seed(seed)
    dt = getattr(torch, dtype)
    n, nv, eps = H * dk, H * dv, 1e-5
    rows = [bf(torch.randn(m, 2 * n + 2 * nv, generator=g)) for m in lens]
    if tweak is not None:
        tweak(rows)
    rot = {"base": 50.0, "dims": rd} if rd else None
    table = sq.build_rot_table(rd, 50.0, max(lens) + 1, device) if rd else None
    state = torch.randn(3, H, dk, dv, generator=g).to(device)
    slots = [2, 0]
    dec = torch.tensor(decay, dtype=torch.float32, device=device)

    def fn(who, sm):
        proj = torch.cat([rows[i][a:a + q] for i, a, q in who]).to(dt).to(device)
        return sq.retention(proj, H, dk, dv, dec, table, rd, eps, state, sm, (min(decay), max(decay)))
    got = in_portions(device, lens, cuts, slots, fn)
    e_out, e_state = 0.0, 0.0
    for i, r in enumerate(rows):
        T = r.shape[0]
        q = orc.rotate_half(r[:, :n].reshape(T, H, dk), torch.arange(T), rot)
        k = orc.rotate_half(r[:, n:2 * n].reshape(T, H, dk), torch.arange(T), rot) * dk ** -0.5
        o, S = orc.retention_core(q, k, r[:, 2 * n:2 * n + nv].reshape(T, H, dv), dec.cpu().to(F64))
        ref = orc.unit_rms(o, eps).reshape(T, nv) * orc.silu(r[:, 2 * n + nv:])
        e_out = max(e_out, float((got[i] - ref).abs().max() / ref.abs().max()))
        e_state = max(e_state, float((state[slots[i]].cpu().to(F64) - S).abs().max() / S.abs().max()))
    return e_out, e_state


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("shape", RET_SHAPES, ids=lambda s: "H%ddk%ddv%drot%d" % s)
@pytest.mark.parametrize("cuts", list(CUTS))
@pytest.mark.parametrize("form", ["default", "segments", "general"])
def test_retention_over_portions_and_slots(device, dtype, shape, cuts, form, monkeypatch):
    """Matrix-core chunks, long portions cut into segments, the general scan and single-token steps; the carried state is
    held to fp32 accuracy also where the rows are bfloat16."""
    if form == "segments":
        monkeypatch.setattr(sq, "CHUNK_FILL_WGS", 4096)
        monkeypatch.setattr(sq, "CHUNK_MIN_SEG", 32)
        monkeypatch.setattr(sq, "CHUNK_MAX_SEGS", 7)
    elif form == "general":
        monkeypatch.setattr(sq, "CHUNK_RECURRENCE", False)
        monkeypatch.setattr(sq, "RECURRENT_STEP", False)
        monkeypatch.setattr(sq, "SCAN_TWO_PASS_MIN", 256)
    H, dk, dv, rd = shape
    decay = [0.999, 0.6, 0.05][:H] if H > 1 else [0.97]
    lens, cc = CUTS[cuts]
    if device == "cpu" and cuts == "long":
        lens, cc = (150, 40), [[3, 90, 1, 17, 39], [20, 1, 2, 1, 16]]
    eo, es = _retention_case(device, dtype, H, dk, dv, rd, lens, cc, decay, dk + dv)
    assert eo < (2e-4 if dtype == "float32" else 8e-3) and es < 5e-5, (eo, es)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("decay", [1.0, 0.02, 0.004, 1e-30], ids=str)
def test_retention_extreme_decays(device, dtype, decay):
    eo, es = _retention_case(device, dtype, 2, 64, 64, 64, (75, 40), [[33, 2, 1, 39], [40]], [decay, 0.98], 5)
    assert eo < (2e-4 if dtype == "float32" else 8e-3) and es < 5e-5, (eo, es)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("back", [0, 1, 15, 16, 17, 31, 32, 33, 64, 200, 399])
@pytest.mark.parametrize("single", [False, True], ids=["prompt", "decoded"])
def test_retention_one_standing_out_key(device, dtype, back, single):
    """The last query lines up with one key (of this chunk, the one before, hundreds of tokens back, its own) whose value is
    far larger than the others': a lost or misplaced key, or a decay applied once too often, moves the output."""
    H, dk, dv, T = 1, 64, 64, 400
    n = H * dk

    def tweak(rows):
        r = rows[0]
        r[:, :2 * n] = bf(r[:, :2 * n] * 0.1)
        j = T - 1 - back
        r[T - 1, :n] = bf(torch.sign(r[T - 1, :n])) * 2
        r[j, n:2 * n] = r[T - 1, :n]
        r[j, 2 * n:2 * n + dv] *= 16
    cuts = [[230, 163] + [1] * 7] if single else [[T]]
    eo, es = _retention_case(device, dtype, H, dk, dv, 0, (T,), cuts, [0.9995], 9, tweak)
    assert eo < (2e-4 if dtype == "float32" else 8e-3) and es < 5e-5, (eo, es)


def _time_mix_case(device, dtype, H, D, lens, cuts, z_of, seed, u_scale=1.0):
    g = torch.Generator().manual_seed(seed)
    dt = getattr(torch, dtype)
    n, eps = H * D, 1e-5
    rows = [bf(torch.randn(m, 5 * n, generator=g)) for m in lens]     # r | k | v | g | z
    w0 = torch.rand(n, generator=g) * 2 - 1
    for r in rows:
        r[:, 4 * n:] = bf(z_of(r[:, 4 * n:]))
    u, nw = torch.randn(n, generator=g) * u_scale, torch.rand(n, generator=g) + 0.5
    state = torch.randn(3, H, D, D, generator=g).to(device)
    slots = [1, 2]
    f = lambda t: t.float().to(device)  # noqa: E731

    def fn(who, sm):
        x = torch.cat([rows[i][a:a + q] for i, a, q in who]).to(dt).to(device)
        r, k, v, gt, z = (x[:, j * n:(j + 1) * n] for j in range(5))
        return sq.time_mix(r, k, v, gt, z, f(w0), f(u), f(nw), eps, H, D, D, state, sm)
    got = in_portions(device, lens, cuts, slots, fn)
    e_out, e_state = 0.0, 0.0
    for i, x in enumerate(rows):
        T = x.shape[0]
        r, k, v, gt, z = (x[:, j * n:(j + 1) * n].reshape(T, H, D) for j in range(5))
        dec = torch.exp(-torch.exp(z.reshape(T, n) + w0.to(F64))).reshape(T, H, D)
        o, S = orc.bonus_core(r, k, v, dec, u.to(F64).reshape(H, D))
        ref = orc.unit_rms(o, eps).reshape(T, n) * nw.to(F64) * orc.silu(gt.reshape(T, n))
        e_out = max(e_out, float((got[i] - ref).abs().max() / ref.abs().max()))
        e_state = max(e_state, float((state[slots[i]].cpu().to(F64) - S).abs().max() / S.abs().max()))
    return e_out, e_state


DECAYS = {"slow": lambda z: z * 0.7 - 4.0, "usual": lambda z: z - 2.5,
          # some channels of some chunks lose everything within a few tokens
          "strong": lambda z: torch.where(z > 1.5, z + 3.0, z - 3.0), "all": lambda z: z * 0.2 + 3.5}


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("shape", [(3, 20), (1, 6), (2, 32), (2, 64), (1, 128), (1, 256), (2, 96)], ids=lambda s: "H%dD%d" % s)
@pytest.mark.parametrize("cuts", list(CUTS))
@pytest.mark.parametrize("form", ["default", "segments", "general"])
def test_time_mixing_over_portions_and_slots(device, dtype, shape, cuts, form, monkeypatch):
    if form == "segments":
        monkeypatch.setattr(sq, "CHUNK_FILL_WGS", 4096)
        monkeypatch.setattr(sq, "CHUNK_MIN_SEG", 32)
        monkeypatch.setattr(sq, "CHUNK_MAX_SEGS", 7)
    elif form == "general":
        monkeypatch.setattr(sq, "CHUNK_RECURRENCE", False)
        monkeypatch.setattr(sq, "RECURRENT_STEP", False)
        monkeypatch.setattr(sq, "SCAN_TWO_PASS_MIN", 256)
    H, D = shape
    lens, cc = CUTS[cuts]
    if device == "cpu" and cuts == "long":
        lens, cc = (150, 40), [[3, 90, 1, 17, 39], [20, 1, 2, 1, 16]]
    for kind in ("usual", "strong"):
        eo, es = _time_mix_case(device, dtype, H, D, lens, cc, DECAYS[kind], D)
        assert eo < (2e-4 if dtype == "float32" else 8e-3) and es < 5e-5, (kind, eo, es)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("kind", list(DECAYS))
@pytest.mark.parametrize("segments", [False, True], ids=["one", "segments"])
def test_time_mixing_decay_ranges(device, dtype, kind, segments, monkeypatch):
    """Decays close to one, usual ones, and channels that are wiped within a token (run token by token inside a chunk)."""
    if segments:
        monkeypatch.setattr(sq, "CHUNK_FILL_WGS", 4096)
        monkeypatch.setattr(sq, "CHUNK_MIN_SEG", 32)
    for D in (32, 64, 128):
        eo, es = _time_mix_case(device, dtype, 2, D, (150, 70), [[129, 1, 20], [70]], DECAYS[kind], 3 + D)
        assert eo < (2e-4 if dtype == "float32" else 8e-3) and es < 5e-5, (D, eo, es)


@pytest.mark.parametrize("device,dtype", CASES)
def test_time_mixing_bonus_counts_for_the_current_token_alone(device, dtype):
    """A bonus so large that it dominates the output: in the state, or on an earlier token, it would show."""
    for cuts in ([[40, 1, 1, 8], [20]], [[1] * 50, [1] * 20]):
        eo, es = _time_mix_case(device, dtype, 2, 32, (50, 20), cuts, DECAYS["usual"], 8, u_scale=100.0)
        assert eo < (2e-4 if dtype == "float32" else 8e-3) and es < 5e-5, (eo, es)


def _window_case(device, dtype, H, G, dk, dv, bs, T, size, single, strong=None):
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(H * 100 + dk + T + size)
    rnd = lambda *s: bf(torch.randn(*s, generator=g))  # noqa: E731
    q, k, v, gate = rnd(T, H, dk), rnd(T, G, dk), rnd(T, G, dv), rnd(T, H + 3)
    eps, scale = 1e-5, 0.4 / dk ** 0.5
    wq, wk = rnd(H * dk) * 0.3 + 1.0, rnd(G * dk) * 0.3 + 1.0
    if strong is not None:
        i, j = strong
        k[j] = q[i, ::H // G] * 1.5
        scale *= 12.0
    f32 = lambda t: t.float().to(device)  # noqa: E731
    qn = (orc.unit_rms(q.reshape(T, -1), eps) * wq).reshape(T, H, dk)
    kn = (orc.unit_rms(k.reshape(T, -1), eps) * wk).reshape(T, G, dk)
    ref = torch.zeros(T, H, dv, dtype=F64)
    for i in range(T):
        lo = max(0, i - size + 1)
        for h in range(H):
            c = h // (H // G)
            ref[i, h] = torch.softmax((kn[lo:i + 1, c] @ qn[i, h]) * scale, 0) @ v[lo:i + 1, c]
    ref = ref * torch.sigmoid(gate[:, :H])[:, :, None]
    pages = torch.randperm(80, generator=g)[:(T + bs - 1) // bs].tolist()
    kc = torch.randn(80 * bs, G * dk, generator=g).to(dt).to(device)      # stale rows everywhere
    vc = torch.randn(80 * bs, G * dv, generator=g).to(dt).to(device)
    out = []
    for ctx, n in ([(0, T)] if not single else [(0, T - 6)] + [(T - 6 + i, 1) for i in range(6)]):
        sm = seq_meta(device, [(0, ctx, n)], bs, [pages])
        src = torch.cat([q[ctx:ctx + n].reshape(n, -1), k[ctx:ctx + n].reshape(n, -1), v[ctx:ctx + n].reshape(n, -1)], 1)
        qq = sq.head_norm_rope_cache(src.to(dt).to(device), H, G, dk, dv, f32(wq), f32(wk), eps, None, 0, sm, kc, vc, dt, whole=True)
        out.append(sq.masked_attention(qq, kc, vc, H, G, dk, dv, sq.MASK_WINDOW, size, scale, None, None, bs, sm,
                                       gate=gate[ctx:ctx + n].to(dt).to(device)))
    return torch.cat(out).float().cpu().reshape(T, H * dv), ref.reshape(T, H * dv)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("shape", [(6, 2, 20, 12), (1, 1, 32, 32), (8, 2, 64, 32), (8, 2, 48, 96), (4, 4, 128, 128), (16, 2, 64, 64)],
                         ids=lambda s: "H%dG%dk%dv%d" % s)
@pytest.mark.parametrize("single", [False, True], ids=["prompt", "decoded"])
@pytest.mark.parametrize("size", [7, 70])
def test_window_attention_alone(device, dtype, shape, single, size):
    got, ref = _window_case(device, dtype, *shape, bs=16, T=75, size=size, single=single)
    assert rel_err(got, ref) < (1e-4 if dtype == "float32" else 4e-2)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("size", [1, 2, 16, 17, 40, 64, 65])
@pytest.mark.parametrize("edge", ["inside", "outside"])
@pytest.mark.parametrize("single", [False, True], ids=["prompt", "decoded"])
def test_window_edge_one_standing_out_key(device, dtype, size, edge, single):
    """The key that stands out for the last query is the oldest one the window keeps, or the one just before it (which must
    stay unseen)."""
    T = 140
    back = size - 1 if edge == "inside" else size
    got, ref = _window_case(device, dtype, 4, 2, 32, 16, 16, T, size, single, strong=(T - 1, T - 1 - back))
    assert rel_err(got[-1:], ref[-1:]) < (1e-4 if dtype == "float32" else 5e-2)
    assert rel_err(got, ref) < (1e-4 if dtype == "float32" else 5e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("T", [1, 7, 16, 17, 33, 64])
@pytest.mark.parametrize("G,K,N", [(4, 64, 32), (4, 96, 48), (3, 256, 80)])
def test_stacked_products_of_short_steps(T, G, K, N):
    """Products with an input and a weight of their own each, in one launch; rows past the step are left alone."""
    g = torch.Generator().manual_seed(T + K)
    w = torch.randn(G, N, K, generator=g).to(torch.bfloat16).cuda()
    tile = sq.stacked_tile(T, K, N, w)
    R = (T + tile - 1) // tile * tile
    x = torch.randn(G, R, K, generator=g).to(torch.bfloat16).cuda()
    y = sq.stacked_linear(x, w, T)
    ref = torch.stack([x[i].cpu().to(F64) @ w[i].cpu().to(F64).T for i in range(G)])
    assert y.shape == (G, R, N) and float((y[:, :T].cpu().to(F64) - ref[:, :T]).abs().max()) < 1e-4 * float(ref.abs().max())


@pytest.mark.parametrize("device", OP_CASES)
@pytest.mark.parametrize("T,E,top,W", [(9, 1, 1, 32), (9, 5, 2, 50), (40, 8, 8, 64), (300, 12, 3, 64), (5, 100, 70, 33),
                                       (20, 16, 4, 4096)])
def test_router_softmax_over_the_chosen(device, T, E, top, W):
    """Weights are the softmax over the chosen logits alone (bias included); logits formed inside the kernel (short steps),
    by a matrix product (long ones), and given."""
    g = torch.Generator().manual_seed(T + E)
    h, w, b = torch.randn(T, W, generator=g), torch.randn(E, W, generator=g) * 2 / math.sqrt(W), torch.randn(E, generator=g) * 2
    z = h.to(F64) @ w.to(F64).T + b.to(F64)
    order = z.topk(top, -1)
    d = lambda t: t.to(device)  # noqa: E731
    for kw in (dict(rows=d(h), router_w=d(w), bias=d(b)), dict(logits=d(z.float()))):
        ids, wts = sq.grouped_router(kw.pop("logits", None), None, 1, 1, top, 1.0, score=sq.SCORE_CHOSEN, rating=sq.RATE_MAX, **kw)
        assert torch.equal(ids.cpu().long().sort(-1).values, order.indices.sort(-1).values)
        ref = torch.softmax(z.gather(1, ids.cpu().long()), -1)
        assert float((wts.cpu().to(F64) - ref).abs().max()) < 1e-5
        assert float((wts.sum(-1) - 1).abs().max()) < 1e-5


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("T,E,top,K,F_", [(7, 5, 2, 40, 24), (50, 1, 1, 32, 16), (300, 3, 3, 64, 48), (700, 4, 1, 96, 64),
                                          (1300, 4, 2, 128, 32), (64, 12, 1, 24, 10), (260, 2, 2, 256, 128)])
def test_silu_gated_experts_and_their_sum(device, dtype, T, E, top, K, F_):
    """Every grouped-GEMM path (16, 32, 64 and 128-row tiles, matrix-core, general, the prompt-sized form) against the dense
    form, and the weighted sum of the chosen rows inside the layer-norm update."""
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(T + E)
    mlp = {"router": {"experts": E, "top": top}, "expert": {"ff": F_}}
    w = {"router": bf(torch.randn(E, K, generator=g) * 3.0 / math.sqrt(K)), "router.b": bf(torch.randn(E, generator=g))}
    for e in range(E):
        for nm, o, i in (("gate", F_, K), ("up", F_, K), ("down", K, F_)):
            w[f"e{e}.{nm}"] = bf(torch.randn(o, i, generator=g) * 1.5 / math.sqrt(i))
    h = bf(torch.randn(T, K, generator=g))
    ref = orc.moe(h, w, "", mlp)
    d32 = lambda t: t.float().to(device)  # noqa: E731
    ids, wts = sq.grouped_router(None, None, 1, 1, top, 1.0, rows=d32(h), router_w=d32(w["router"]), score=sq.SCORE_CHOSEN,
                                 rating=sq.RATE_MAX, bias=d32(w["router.b"]))
    w13 = torch.stack([torch.cat([w[f"e{e}.gate"], w[f"e{e}.up"]]) for e in range(E)]).to(dt).to(device)
    w2 = torch.stack([w[f"e{e}.down"] for e in range(E)]).to(dt).to(device)
    y = sq.routed_experts(h.to(dt).to(device), w13, w2, ids, wts, sq.GLU_SILU)
    assert rel_err(y, ref) < (1e-4 if dtype == "float32" else 3e-2)
    rows = sq.routed_experts(h.to(dt).to(device), w13, w2, ids, wts, sq.GLU_SILU, combine=False)
    nw = torch.rand(K, generator=g) + 0.5
    x = torch.randn(T, K, generator=g)
    xs = x.clone().to(device)
    sq.layer_norm_residual(xs, rows, nw.to(device), 1e-5, torch.float32)
    assert rel_err(xs, x.to(F64) + orc.layer_norm(ref, nw.to(F64), 1e-5)) < (1e-4 if dtype == "float32" else 3e-2)
    gu = torch.randn(T, 2 * F_, generator=g).to(dt)
    a = sq.glu_act(gu.to(device), sq.GLU_SILU)
    r = orc.silu(gu[:, :F_].to(F64)) * gu[:, F_:].to(F64)
    assert rel_err(a, r) < (1e-5 if dtype == "float32" else 1e-2)


# ---------------------------------------------------------------------------------- random configurations
def _random_config(rng):
    W = rng.choice([64, 96, 160])

    def ret():
        H, dk = rng.choice([1, 2, 3]), rng.choice([16, 32, 64, 96])
        m = {"heads": H, "dim": dk, "vdim": rng.choice([16, 24, 64, 96]),
             "decay": [round(1 - 2.0 ** -rng.choice([1, 4, 6, 9]), 6) for _ in range(H)]}
        rd = rng.choice([0, 2, dk // 2 // 2 * 2, dk])
        if rd:
            m["rot"] = {"base": rng.choice([100.0, 10000.0]), "dims": rd}
        return m

    def par():
        G, dk = rng.choice([1, 2]), rng.choice([16, 32, 48, 64])
        return {"left": {"heads": G * rng.choice([1, 2, 4]), "kv_heads": G, "dim": dk, "vdim": rng.choice([16, 32, 48]),
                         "scale": round(dk ** -0.5, 6), "mask": {"size": rng.choice([1, 3, 16, 30, 64, 100])}},
                "right": {"heads": rng.choice([1, 2, 3]), "dim": rng.choice([8, 32, 48, 64]), "decay_rank": rng.choice([2, 16])},
                "left_scale": rng.choice([1.0, 0.3, -0.8]), "right_scale": rng.choice([1.0, 1.7, 0.4])}
    layers = []
    for _ in range(rng.choice([2, 3, 4, 5])):
        t = rng.choice(["retention", "parallel"])
        E = rng.choice([1, 2, 8, 12])
        k = rng.random()
        mlp = None if k < 0.2 else {"kind": "dense", "ff": rng.choice([48, 64, 100])} if k < 0.6 else \
            {"kind": "moe", "expert": {"ff": rng.choice([16, 32, 40])}, "router": {"experts": E, "top": rng.randrange(1, min(E, 3) + 1)}}
        layers.append({"type": t, "mixer": ret() if t == "retention" else par(), "mlp": mlp})
    return {"architecture": "Bazurax", "width": W, "vocab": rng.choice([97, 300]), "norm": {"eps": rng.choice([1e-5, 1e-6])},
            "layers": layers}


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("seed", [3, 14, 15, 92, 65])
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
        lg, o = eng.score_step(entries, ["r%d" % i for i, _ in who if at[i] == lens[i]]), 0
        for i, n in who:
            got[i].append(lg[o:o + n])
            o += n
    for i in range(4):
        assert close(torch.cat(got[i], 0), refs[i], dtype), (i, cfg)
    assert eng.sched.num_used_blocks() == 0
