"""Helpers of the layer-list model tests: engines on small pools, portions, per-sequence step metadata, error measures."""
import torch

from xgserve.engine import EngineConfig, LLMEngine
from xgserve.ops import seqmix as sq

F64 = torch.float64
TOL = {"float32": 2e-4, "bfloat16": 6e-2}


def engine(path, device, dtype, **kw):
    args = dict(model=path, checkpoint=path, device=device, dtype=dtype, block_size=4, num_blocks=64, max_num_seqs=3,
                max_num_batched_tokens=256, max_model_len=200, use_graphs=False, enable_prefix_cache=False)
    args.update(kw)
    return LLMEngine(EngineConfig(**args))


def tokens_of(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def row_errs(got, ref):
    """Per row: root mean square of the difference over that of the reference, means taken off."""
    got, ref = got.detach().to("cpu", F64), ref.to(F64)
    d = got - ref
    d = d - d.mean(-1, keepdim=True)
    r = ref - ref.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / r.pow(2).mean(-1).sqrt()


def rel_err(got, ref):
    return float(row_errs(got, ref).max())


def close(got, ref, dtype):
    """float32: every position within 2e-4. bfloat16: rounding can tip a router's close call at a token, whose
    feed-forward output is then another one altogether, and later tokens see it through the cache. So a few positions
    may exceed the rounding level while most stay within it; a wrong mechanism is caught by the float32 runs and moves
    most positions."""
    e = row_errs(got, ref)
    if dtype == "float32":
        return float(e.max()) < TOL[dtype]
    return bool(torch.isfinite(e).all()) and float((e > TOL[dtype]).double().mean()) <= 0.15 and \
        float(e.median()) < TOL[dtype] / 2


def run_portions(eng, rid, toks, portions):
    """Feed `toks` in the given portion sizes (the rest one by one); logits of every position."""
    out, at = [], 0
    sizes = list(portions)
    while at < len(toks):
        n = min(sizes.pop(0) if sizes else 1, len(toks) - at)
        end = [rid] if at + n == len(toks) else []
        out.append(eng.score_step([(rid, toks[at:at + n], list(range(n)))], end))
        at += n
    return torch.cat(out, 0)


def seq_meta(device, rows, block_size, tables):
    """rows: [(slot, context length, tokens in this step)] -> SeqMeta; tables: page list per row."""
    qsl, sl, slots, tseq, pos, smap = [0], [], [], [], [], []
    width = max(len(t) for t in tables)
    for i, (slot, ctx, q) in enumerate(rows):
        qsl.append(qsl[-1] + q)
        sl.append(ctx + q)
        slots.append(slot)
        for p in range(ctx, ctx + q):
            tseq.append(i)
            pos.append(p)
            smap.append(tables[i][p // block_size] * block_size + p % block_size)
    bt = [t + [0] * (width - len(t)) for t in tables]
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)  # noqa: E731
    return sq.SeqMeta(len(rows), max(r[2] for r in rows), i32(qsl), i32(sl), i32(slots), i32(bt), i32(tseq), i32(pos),
                      i32(smap))
