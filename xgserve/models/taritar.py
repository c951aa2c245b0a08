"""Taritar: a pre-norm decoder with several residual streams and shared key / value caches, on the paged engine.

    x_s = embed[token] * c + pos[position]      for every stream s = 1 .. S          (c = cfg.embed_scale)
    per sublayer f (mixer, then feed-forward) with its own weights a [S], b [S], M [S, S]:
        u   = sum_s a[s] x_s
        x_t <- sum_s M[s, t] x_s + b[t] f(N(u))           (all streams from the old ones)
    logits = cap(W_head N(sum_s x_s)),          cap(z) = c tanh(z / c)               (c = cfg.logit_softcap)

N is the RMS norm with a plain weight. The streams are fp32 throughout; mixing them, adding a sublayer's output, the next
sublayer's weighted sum and its norm run in one kernel (ops.seqmix.hyper_residual).

  * `WindowKeepAttention`: grouped-query attention, the first rot.dims entries of each head rotated in (2i, 2i + 1)
    pairs; scores bounded by cap(.); a sliding window that also keeps the sequence's first `keep_first` tokens. A layer
    with `kv_from` has queries only and reads the cached keys and values of that earlier layer (its LayerCache holds
    the owner's tensors).
  * Feed-forward: `GatedMLP` with the clamped GLU, `SoftmaxRouterMoE` (softmax scores over all experts, groups rated by
    their best member, the scores as weights, a shared expert times a sigmoid gate per token), or none.

Everything a sequence carries between steps is in its pages, so prompts can share prefixes and drafts can be rolled back.
"""
from __future__ import annotations

import math
from typing import Dict, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from ..ops import seqmix as sq
from ..parallel.state import get_state
from .base import AttnMeta
from .config import ModelConfig
from .seq_cache import LayerCache, SeqCache
from .vizonex import GLU_ALPHA, GatedMLP


def _p(t):
    return nn.Parameter(t, requires_grad=False)


class HyperConnection(nn.Module):
    """Weights of one sublayer's connection to the residual streams: read, write, mix [from, to]."""

    def __init__(self, streams: int, device):
        super().__init__()
        f = lambda *s: torch.zeros(*s, device=device, dtype=torch.float32)  # noqa: E731
        self.w_in, self.w_out, self.mix = _p(f(streams)), _p(f(streams)), _p(f(streams, streams))


class WindowKeepAttention(nn.Module):
    def __init__(self, width: int, m: dict, device, dtype):
        super().__init__()
        e = lambda *s: torch.empty(*s, device=device, dtype=dtype)  # noqa: E731
        self.H, self.G, self.dk, self.dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
        self.scale, self.softcap = float(m["scale"]), float(m.get("softcap") or 0.0)
        mask = m.get("mask")
        self.mask, self.size, self.keep = (sq.MASK_WINDOW, int(mask["size"]), int(mask.get("keep_first", 0))) if mask \
            else (sq.MASK_CAUSAL, 0, 0)
        self.rot = m.get("rot") or None
        self.rot_dims = int(self.rot["dims"]) if self.rot else 0
        self.kv_from = m.get("kv_from")
        self.nq, self.nk, self.nv = self.H * self.dk, self.G * self.dk, self.G * self.dv
        own = self.kv_from is None
        self.in_proj = _p(e(self.nq + (self.nk + self.nv if own else 0), width))   # fused rows [q | k | v], or [q]
        self.o = _p(e(width, self.H * self.dv))

    def forward(self, h, sm: sq.SeqMeta, lc: LayerCache, block_size: int, rot):
        proj = F.linear(h, self.in_proj)
        if self.kv_from is None:
            q = sq.head_norm_rope_cache(proj, self.H, self.G, self.dk, self.dv, None, None, 0.0, rot, self.rot_dims, sm,
                                        lc.k, lc.v, h.dtype)
        elif rot is not None:
            q = sq.head_norm_rope_cache(proj, self.H, 0, self.dk, self.dv, None, None, 0.0, rot, self.rot_dims, sm, None,
                                        None, h.dtype)
        else:
            q = proj
        o = sq.masked_attention(q, lc.k, lc.v, self.H, self.G, self.dk, self.dv, self.mask, self.size, self.scale, None,
                                None, block_size, sm, softcap=self.softcap, keep_first=self.keep)
        return F.linear(o, self.o)


class SoftmaxRouterMoE(nn.Module):
    def __init__(self, width: int, mlp: dict, device, dtype):
        super().__init__()
        r = mlp["router"]
        g = r.get("groups") or {"count": 1, "keep": 1}
        self.E, self.top, self.count, self.keep = int(r["experts"]), int(r["top"]), int(g["count"]), int(g["keep"])
        self.ff, self.limit = int(mlp["expert"]["ff"]), float(mlp["expert"]["limit"])
        self.w13 = _p(torch.empty(self.E, 2 * self.ff, width, device=device, dtype=dtype))  # per expert rows [gate | up]
        self.w2 = _p(torch.empty(self.E, width, self.ff, device=device, dtype=dtype))
        sh = mlp.get("shared")
        self.shared = GatedMLP(width, sh["ff"], sq.GLU_CLAMPED, sh["limit"], device, dtype) if sh else None
        # router rows, then (with a shared expert) the row of its gate
        self.router = _p(torch.zeros(self.E + (1 if sh else 0), width, device=device, dtype=torch.float32))

    def forward(self, n32, nact):
        """(shared expert's output or None, its gate per token or None, the routed experts' rows)."""
        ids, wts, gate = sq.grouped_router(None, None, self.count, self.keep, self.top, 1.0, rows=n32, router_w=self.router,
                                           score=sq.SCORE_SOFTMAX, rating=sq.RATE_MAX, extra_gate=self.shared is not None,
                                           want_gate=True)
        y3 = sq.routed_experts(nact, self.w13, self.w2, ids, wts, sq.GLU_CLAMPED, self.limit, GLU_ALPHA, combine=False)
        return (self.shared(nact) if self.shared is not None else None), gate, y3


class TaritarLayer(nn.Module):
    def __init__(self, cfg: ModelConfig, spec: dict, device, dtype):
        super().__init__()
        W = cfg.hidden_size
        f = lambda *s: torch.zeros(*s, device=device, dtype=torch.float32)  # noqa: E731
        self.mix = WindowKeepAttention(W, spec["mixer"], device, dtype)
        self.norm1, self.hc1 = _p(f(W)), HyperConnection(cfg.streams, device)
        mlp = spec.get("mlp")
        self.mlp, self.moe = None, False
        if mlp is not None:
            self.norm2, self.hc2 = _p(f(W)), HyperConnection(cfg.streams, device)
            self.moe = mlp["kind"] == "moe"
            self.mlp = SoftmaxRouterMoE(W, mlp, device, dtype) if self.moe else \
                GatedMLP(W, mlp["ff"], sq.GLU_CLAMPED, mlp["limit"], device, dtype)


class TaritarForCausalLM(nn.Module):
    needs_seq_meta = True       # every operator takes the step's per-sequence metadata; nothing is kept per slot

    def __init__(self, cfg: ModelConfig, device="cpu", dtype=torch.bfloat16, tp: Optional[int] = None,
                 rank: Optional[int] = None):
        super().__init__()
        tp = get_state().tp_size if tp is None else tp
        if tp != 1:
            raise ValueError("Taritar runs with tp=1 (use DP replicas to scale)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Taritar runs in bfloat16 or float32")
        self.cfg, self.tp, self.rank = cfg, 1, 0
        self.device, self.dtype = torch.device(device), dtype
        W = cfg.hidden_size
        self.embed = _p(torch.empty(cfg.vocab_size, W, device=device, dtype=dtype))
        self.pos = _p(torch.empty(cfg.max_position, W, device=device, dtype=dtype))
        self.layers = nn.ModuleList([TaritarLayer(cfg, spec, device, dtype) for spec in cfg.layer_specs])
        self.final_norm = _p(torch.zeros(W, device=device, dtype=torch.float32))
        self.head = _p(torch.empty(cfg.vocab_size, W, device=device, dtype=dtype))
        self.num_kv_heads_local = 1
        self._rot: Dict[tuple, torch.Tensor] = {}
        self._rot_len = 0
        self.set_max_positions(min(cfg.max_position, 4096))
        self.keep_residuals = None   # tests: a list that collects the sum of the streams after every layer

    # ------------------------------------------------------------------ positions
    def set_max_positions(self, n: int) -> None:
        """(Re)build the rotation tables for positions [0, n) -- the runner passes its max_model_len."""
        if n <= self._rot_len:
            return
        self._rot = {}
        for L in self.layers:
            key = self._rot_key(L.mix)
            if key is not None and key not in self._rot:
                self._rot[key] = sq.build_rot_table(key[0], key[1], n, self.device)
        self._rot_len = n

    @staticmethod
    def _rot_key(a: WindowKeepAttention):
        return (a.rot_dims, float(a.rot["base"])) if a.rot_dims else None

    # ------------------------------------------------------------------ cache
    def alloc_cache(self, num_blocks: int, block_size: int, max_num_seqs: int) -> SeqCache:
        sc = SeqCache(block_size=block_size)
        rows = num_blocks * block_size
        for L in self.layers:
            a = L.mix
            if a.kv_from is None:
                sc.layers.append(LayerCache(k=torch.zeros(rows, a.nk, dtype=self.dtype, device=self.device),
                                            v=torch.zeros(rows, a.nv, dtype=self.dtype, device=self.device)))
            else:   # the owner's pages
                o = sc.layers[a.kv_from]
                sc.layers.append(LayerCache(k=o.k, v=o.v))
        return sc

    def cache_bytes_per_block(self, block_size: int) -> int:
        esz = torch.tensor([], dtype=self.dtype).element_size()
        return block_size * sum((L.mix.nk + L.mix.nv) * esz for L in self.layers if L.mix.kv_from is None)

    # ------------------------------------------------------------------ weights
    @torch.no_grad()
    def random_init(self, seed: int = 0):
        g = torch.Generator().manual_seed(seed)

        def mat(p, gain=1.0):
            p.copy_((torch.randn(p.shape, generator=g) * gain / math.sqrt(p.shape[-1])).to(p.dtype))

        def vec(p, std, mean=0.0):
            p.copy_((torch.randn(p.shape, generator=g) * std + mean).to(p.dtype))

        def hyper(hc):
            S = hc.w_in.numel()
            vec(hc.w_in, 0.1, 1.0 / S)
            vec(hc.w_out, 0.2, 1.0)
            hc.mix.copy_(0.9 * torch.eye(S) + torch.randn(S, S, generator=g) * 0.1 / S)
        self.embed.copy_((torch.randn(self.embed.shape, generator=g) * 0.3).to(self.dtype))
        self.pos.copy_((torch.randn(self.pos.shape, generator=g) * 0.1).to(self.dtype))
        mat(self.head)
        vec(self.final_norm, 0.1, 1.0)
        for L in self.layers:
            vec(L.norm1, 0.1, 1.0)
            hyper(L.hc1)
            mat(L.mix.in_proj)
            mat(L.mix.o)
            if L.mlp is None:
                continue
            vec(L.norm2, 0.1, 1.0)
            hyper(L.hc2)
            if L.moe:
                mat(L.mlp.router, 2.0)
                mat(L.mlp.w13)
                mat(L.mlp.w2)
            dense = L.mlp.shared if L.moe else L.mlp
            if dense is not None:
                mat(dense.gate_up)
                mat(dense.down)

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids: torch.Tensor, meta: AttnMeta, cache: SeqCache):
        sm = meta.seq
        if sm is None:
            raise ValueError("Taritar needs the step's per-sequence metadata (AttnMeta.seq)")
        eps, dt, S, last, keep = self.cfg.norm_eps, self.dtype, self.cfg.streams, len(self.layers) - 1, self.keep_residuals
        x = sq.embed_rows(input_ids, self.embed, self.pos, sm.positions, self.cfg.embed_scale)
        first = self.layers[0]
        x, n32, n = sq.hyper_residual(x, S, None, None, None, None, first.hc1.w_in, first.norm1, eps, dt)
        for i, (L, lc) in enumerate(zip(self.layers, cache.layers)):
            # what reads the streams next: the next layer's mixer, or the sum for the head
            nxt = (self.layers[i + 1].hc1.w_in, self.layers[i + 1].norm1) if i < last else (None, self.final_norm)
            after = (L.hc2.w_in, L.norm2) if L.mlp is not None else nxt
            y = L.mix(n, sm, lc, cache.block_size, self._rot.get(self._rot_key(L.mix)))
            x, n32, n = sq.hyper_residual(x, S, y, None, L.hc1.w_out, L.hc1.mix, *after, eps, dt, want_f32=L.moe,
                                          store=L.mlp is not None or i < last or keep is not None)
            if L.mlp is not None:
                y1, gate, y3 = L.mlp(n32, n) if L.moe else (L.mlp(n), None, None)
                x, n32, n = sq.hyper_residual(x, S, y1, y3, L.hc2.w_out, L.hc2.mix, *nxt, eps, dt, y_gate=gate,
                                              store=i < last or keep is not None)
            if keep is not None:
                keep.append(x.sum(1))
        return n

    def compute_logits(self, h: torch.Tensor) -> torch.Tensor:
        logits = F.linear(h, self.head)
        return sq.soft_cap_(logits, self.cfg.logit_softcap) if self.cfg.logit_softcap else logits

    def set_moe_comm(self, mode: str):
        pass


def count_params(cfg: ModelConfig) -> int:
    W, V, S = cfg.hidden_size, cfg.vocab_size, cfg.streams
    hc = S * (S + 2)
    n = 2 * V * W + W + cfg.max_position * W
    for spec in cfg.layer_specs:
        m, mlp = spec["mixer"], spec.get("mlp")
        n += W + hc + m["heads"] * (m["dim"] + m["vdim"]) * W
        if m.get("kv_from") is None:
            n += m["kv_heads"] * (m["dim"] + m["vdim"]) * W
        if mlp is None:
            continue
        n += W + hc
        if mlp["kind"] == "dense":
            n += 3 * W * mlp["ff"]
            continue
        E = mlp["router"]["experts"]
        n += E * W + 3 * E * W * mlp["expert"]["ff"]
        if mlp.get("shared"):
            n += 3 * W * mlp["shared"]["ff"] + W
    return n
