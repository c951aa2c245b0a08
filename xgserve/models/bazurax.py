"""Bazurax: a decoder that norms every sublayer's output before it joins the residual, on the paged / slotted engine.

    x_0 = L(embed[token]; embed.norm)
    x  <- x + L(mixer(x); norm1);   x <- x + L(ff(x); norm2)          logits = embed L(x; final.norm)
    L(v; w) = (v - mean) / sqrt(variance + eps) * w

The sublayers read x itself. The residual stream x is fp32 throughout; a sublayer's output norm, the residual sum and the
activation copy of the new x (what the next sublayer reads) are one kernel.

Mixers (reusable modules, every constant a parameter):
  * `Retention` ("retention"): linear attention with one constant decay per head, S <- decay_h S + k v^T, o = S^T q on an
    fp32 [dim x vdim] state per head and slot; q and k rotated in (i, i + dims / 2) pairs; each head's o divided by its root
    mean square, times silu(W_g h).
  * `ParallelMixer` ("parallel"): left_scale * left + right_scale * right of two branches reading the same input. Left,
    `WholeNormWindowAttention`: grouped-query attention without positions in a sliding window, q / k RMS-normed over their
    whole projections, one output gate per head. Right, `TimeMix`: every projection reads its own mix of the token's and the
    previous token's input; a decay per key channel from a low-rank projection, w = exp(-exp(.)); a bonus for the current
    token; o RMS-normed per head, times a weight and a gate.
Feed-forward: `GatedMLP` with a silu gate, `ChosenSoftmaxMoE` (router logits with a bias, the `top` largest weighted by the
softmax over the chosen logits alone), or none.

What a sequence carries between steps (ModelRunner allocates it through alloc_cache): K / V pages of the left branches; per
state slot the recurrent states and the time-mixing layers' last input row.
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
from .vizonex import GatedMLP


def _p(t):
    return nn.Parameter(t, requires_grad=False)


class Retention(nn.Module):
    def __init__(self, width: int, m: dict, eps: float, device, dtype):
        super().__init__()
        self.H, self.dk, self.dv, self.eps = int(m["heads"]), int(m["dim"]), int(m["vdim"]), eps
        self.n, self.nv = self.H * self.dk, self.H * self.dv
        self.rot = m.get("rot") or None
        self.rot_dims = int(self.rot["dims"]) if self.rot else 0
        self.decay_range = (min(float(a) for a in m["decay"]), max(float(a) for a in m["decay"]))
        self.register_buffer("decay", torch.tensor([float(a) for a in m["decay"]], dtype=torch.float32, device=device))
        self.in_proj = _p(torch.empty(2 * self.n + 2 * self.nv, width, device=device, dtype=dtype))   # rows [q | k | v | g]
        self.o = _p(torch.empty(width, self.nv, device=device, dtype=dtype))

    def rot_key(self):
        return (self.rot_dims, float(self.rot["base"])) if self.rot_dims else None

    def forward(self, h, sm: sq.SeqMeta, lc: LayerCache, rot):
        y = sq.retention(F.linear(h, self.in_proj), self.H, self.dk, self.dv, self.decay, rot, self.rot_dims, self.eps,
                         lc.gla, sm, self.decay_range)
        return F.linear(y, self.o)


class WholeNormWindowAttention(nn.Module):
    def __init__(self, width: int, m: dict, eps: float, device, dtype):
        super().__init__()
        f = lambda *s: torch.zeros(*s, device=device, dtype=torch.float32)  # noqa: E731
        self.H, self.G, self.dk, self.dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
        self.scale, self.eps = float(m["scale"]), eps
        mask = m.get("mask")
        self.mask, self.size = (sq.MASK_WINDOW, int(mask["size"])) if mask else (sq.MASK_CAUSAL, 0)
        self.nq, self.nk, self.nv = self.H * self.dk, self.G * self.dk, self.G * self.dv
        self.ch = self.nq + self.nk + self.nv
        self.in_proj = _p(torch.empty(self.ch + self.H, width, device=device, dtype=dtype))   # rows [q | k | v | gate]
        self.q_norm, self.k_norm = _p(f(self.nq)), _p(f(self.nk))
        self.o = _p(torch.empty(width, self.H * self.dv, device=device, dtype=dtype))

    def forward(self, h, sm: sq.SeqMeta, lc: LayerCache, block_size: int):
        proj = F.linear(h, self.in_proj)
        q = sq.head_norm_rope_cache(proj, self.H, self.G, self.dk, self.dv, self.q_norm, self.k_norm, self.eps, None, 0, sm,
                                    lc.k, lc.v, h.dtype, whole=True)
        o = sq.masked_attention(q, lc.k, lc.v, self.H, self.G, self.dk, self.dv, self.mask, self.size, self.scale, None, None,
                                block_size, sm, gate=proj[:, self.ch:])
        return F.linear(o, self.o)


class TimeMix(nn.Module):
    def __init__(self, width: int, m: dict, eps: float, device, dtype):
        super().__init__()
        e = lambda *s: torch.empty(*s, device=device, dtype=dtype)  # noqa: E731
        f = lambda *s: torch.zeros(*s, device=device, dtype=torch.float32)  # noqa: E731
        self.H, self.dk, self.eps, self.rank = int(m["heads"]), int(m["dim"]), eps, int(m["decay_rank"])
        self.n = self.H * self.dk
        self.mu = _p(f(5, width))                 # shares of the previous token in the inputs of r, k, v, g, w
        self.rkvg = _p(e(4, self.n, width))
        self.w1, self.w2, self.w0 = _p(e(self.rank, width)), _p(e(self.n, self.rank)), _p(f(self.n))
        self.u, self.norm = _p(f(self.n)), _p(f(self.n))
        self.o = _p(e(width, self.n))

    def forward(self, x, sm: sq.SeqMeta, lc: LayerCache, dtype):
        """x: the fp32 mixer input (the mixes are formed before they are rounded)."""
        T = x.shape[0]
        tile = sq.stacked_tile(T, x.shape[1], self.n, self.rkvg) if sm.max_q == 1 else 0
        mixed = sq.token_shift_mix(x, self.mu, lc.shift, sm, dtype, tile or 1)
        if tile:   # single tokens: the four products in one launch
            r, k, v, g = sq.stacked_linear(mixed[:4], self.rkvg, T)[:, :T].unbind(0)
        else:
            r, k, v, g = (F.linear(mixed[j], self.rkvg[j]) for j in range(4))
        z = F.linear(sq.tanh_cols(F.linear(mixed[4][:T], self.w1), 0, self.rank), self.w2)
        y = sq.time_mix(r, k, v, g, z, self.w0, self.u, self.norm, self.eps, self.H, self.dk, self.dk, lc.gla, sm,
                        dtype)
        return F.linear(y, self.o)


class ParallelMixer(nn.Module):
    def __init__(self, width: int, m: dict, eps: float, device, dtype):
        super().__init__()
        self.left = WholeNormWindowAttention(width, m["left"], eps, device, dtype)
        self.right = TimeMix(width, m["right"], eps, device, dtype)
        self.scales = (float(m["left_scale"]), float(m["right_scale"]))

    def forward(self, x, h, sm: sq.SeqMeta, lc: LayerCache, block_size: int):
        """The two branch outputs; their weighted sum is formed by the residual update."""
        return self.left(h, sm, lc, block_size), self.right(x, sm, lc, h.dtype)


class ChosenSoftmaxMoE(nn.Module):
    def __init__(self, width: int, mlp: dict, device, dtype):
        super().__init__()
        self.E, self.top = int(mlp["router"]["experts"]), int(mlp["router"]["top"])
        self.ff = int(mlp["expert"]["ff"])
        self.router = _p(torch.zeros(self.E, width, device=device, dtype=torch.float32))
        self.router_b = _p(torch.zeros(self.E, device=device, dtype=torch.float32))
        self.w13 = _p(torch.empty(self.E, 2 * self.ff, width, device=device, dtype=dtype))   # per expert rows [gate | up]
        self.w2 = _p(torch.empty(self.E, width, self.ff, device=device, dtype=dtype))

    def forward(self, x, h):
        """The experts' output rows; the residual update sums them per token."""
        ids, wts = sq.grouped_router(None, None, 1, 1, self.top, 1.0, rows=x, router_w=self.router, score=sq.SCORE_CHOSEN,
                                     rating=sq.RATE_MAX, bias=self.router_b)
        return sq.routed_experts(h, self.w13, self.w2, ids, wts, sq.GLU_SILU, combine=False)


class BazuraxLayer(nn.Module):
    def __init__(self, cfg: ModelConfig, spec: dict, device, dtype):
        super().__init__()
        W = cfg.hidden_size
        f = lambda *s: torch.zeros(*s, device=device, dtype=torch.float32)  # noqa: E731
        self.kind, self.eps = spec["type"], cfg.norm_eps
        self.mix = (Retention if self.kind == "retention" else ParallelMixer)(W, spec["mixer"], cfg.norm_eps, device, dtype)
        self.norm1 = _p(f(W))
        mlp = spec.get("mlp")
        self.mlp, self.moe = None, False
        if mlp is not None:
            self.norm2 = _p(f(W))
            self.moe = mlp["kind"] == "moe"
            self.mlp = ChosenSoftmaxMoE(W, mlp, device, dtype) if self.moe else \
                GatedMLP(W, mlp["ff"], sq.GLU_SILU, 0.0, device, dtype)

    def forward(self, x, h, sm: sq.SeqMeta, lc: LayerCache, block_size: int, rot, next_w):
        """x: fp32 residual (updated in place), h: x as an activation tensor. Returns the new h, or with `next_w` the layer
        norm of the new x."""
        dt, last = h.dtype, self.mlp is None
        nw = next_w if last else None
        if self.kind == "retention":
            _, h = sq.layer_norm_residual(x, self.mix(h, sm, lc, rot), self.norm1, self.eps, dt, next_w=nw)
        else:
            ya, yb = self.mix(x, h, sm, lc, block_size)
            _, h = sq.layer_norm_residual(x, ya, self.norm1, self.eps, dt, y2=yb, scales=self.mix.scales, next_w=nw)
        if not last:
            y = self.mlp(x, h) if self.moe else self.mlp(h)
            _, h = sq.layer_norm_residual(x, y, self.norm2, self.eps, dt, next_w=next_w)
        return h


class BazuraxForCausalLM(nn.Module):
    has_sequence_state = True   # recurrent state per slot: no prefix reuse, no draft verification

    def __init__(self, cfg: ModelConfig, device="cpu", dtype=torch.bfloat16, tp: Optional[int] = None,
                 rank: Optional[int] = None):
        super().__init__()
        tp = get_state().tp_size if tp is None else tp
        if tp != 1:
            raise ValueError("Bazurax runs with tp=1 (use DP replicas to scale)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Bazurax runs in bfloat16 or float32")
        self.cfg, self.tp, self.rank = cfg, 1, 0
        self.device, self.dtype = torch.device(device), dtype
        W = cfg.hidden_size
        f = lambda *s: torch.zeros(*s, device=device, dtype=torch.float32)  # noqa: E731
        self.embed = _p(torch.empty(cfg.vocab_size, W, device=device, dtype=dtype))   # also the output matrix
        self.embed_norm, self.final_norm = _p(f(W)), _p(f(W))
        self.layers = nn.ModuleList([BazuraxLayer(cfg, spec, device, dtype) for spec in cfg.layer_specs])
        self.num_kv_heads_local = 1
        self._rot: Dict[tuple, torch.Tensor] = {}
        self._rot_len = 0
        self.set_max_positions(min(cfg.max_position, 4096))
        self.keep_residuals = None   # tests: a list that collects x after every layer

    # ------------------------------------------------------------------ positions
    def set_max_positions(self, n: int) -> None:
        """(Re)build the rotation tables for positions [0, n) -- the runner passes its max_model_len."""
        if n <= self._rot_len:
            return
        self._rot = {}
        for L in self.layers:
            key = L.mix.rot_key() if L.kind == "retention" else None
            if key is not None and key not in self._rot:
                self._rot[key] = sq.build_rot_table(key[0], key[1], n, self.device)
        self._rot_len = n

    # ------------------------------------------------------------------ cache / state
    def alloc_cache(self, num_blocks: int, block_size: int, max_num_seqs: int) -> SeqCache:
        dev = self.device
        f32 = dict(dtype=torch.float32, device=dev)
        sc = SeqCache(block_size=block_size)
        rows = num_blocks * block_size
        for L in self.layers:
            lc = LayerCache()
            if L.kind == "retention":
                m = L.mix
                lc.gla = torch.zeros(max_num_seqs, m.H, m.dk, m.dv, **f32)
            else:
                a, r = L.mix.left, L.mix.right
                lc.k = torch.zeros(rows, a.nk, dtype=self.dtype, device=dev)
                lc.v = torch.zeros(rows, a.nv, dtype=self.dtype, device=dev)
                lc.gla = torch.zeros(max_num_seqs, r.H, r.dk, r.dk, **f32)
                lc.shift = torch.zeros(max_num_seqs, self.cfg.hidden_size, **f32)
            sc.layers.append(lc)
        return sc

    def cache_bytes_per_block(self, block_size: int) -> int:
        esz = torch.tensor([], dtype=self.dtype).element_size()
        return max(1, block_size * sum((L.mix.left.nk + L.mix.left.nv) * esz for L in self.layers if L.kind == "parallel"))

    def state_bytes_per_slot(self) -> int:
        n = 0
        for L in self.layers:
            if L.kind == "retention":
                n += L.mix.H * L.mix.dk * L.mix.dv
            else:
                n += L.mix.right.H * L.mix.right.dk ** 2 + self.cfg.hidden_size
        return 4 * n

    # ------------------------------------------------------------------ weights
    @torch.no_grad()
    def random_init(self, seed: int = 0):
        g = torch.Generator().manual_seed(seed)

        def mat(p, gain=1.0):
            p.copy_((torch.randn(p.shape, generator=g) * gain / math.sqrt(p.shape[-1])).to(p.dtype))

        def vec(p, std, mean=0.0):
            p.copy_((torch.randn(p.shape, generator=g) * std + mean).to(p.dtype))
        mat(self.embed)
        vec(self.embed_norm, 0.1, 1.0)
        vec(self.final_norm, 0.1, 1.0)
        for L in self.layers:
            vec(L.norm1, 0.1, 1.0)
            if L.kind == "retention":
                mat(L.mix.in_proj)
                mat(L.mix.o)
            else:
                a, r = L.mix.left, L.mix.right
                mat(a.in_proj)
                vec(a.q_norm, 0.1, 1.0)
                vec(a.k_norm, 0.1, 1.0)
                mat(a.o)
                r.mu.copy_(torch.rand(r.mu.shape, generator=g))
                for p in (r.rkvg, r.w1, r.w2, r.o):
                    mat(p)
                r.w0.copy_(torch.rand(r.n, generator=g) * 5.0 - 6.0)
                vec(r.u, 0.5)
                vec(r.norm, 0.1, 1.0)
            if L.mlp is not None:
                vec(L.norm2, 0.1, 1.0)
                if L.moe:
                    mat(L.mlp.router, 2.0)
                    vec(L.mlp.router_b, 0.3)
                    mat(L.mlp.w13)
                    mat(L.mlp.w2)
                else:
                    mat(L.mlp.gate_up)
                    mat(L.mlp.down)

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids: torch.Tensor, meta: AttnMeta, cache: SeqCache):
        sm = meta.seq
        if sm is None:
            raise ValueError("Bazurax needs the step's per-sequence metadata (AttnMeta.seq)")
        x, h = sq.layer_norm_residual(None, self.embed, self.embed_norm, self.cfg.norm_eps, self.dtype, ids=input_ids)
        last, keep = len(self.layers) - 1, self.keep_residuals
        for i, (L, lc) in enumerate(zip(self.layers, cache.layers)):
            rot = self._rot.get(L.mix.rot_key()) if L.kind == "retention" else None
            h = L(x, h, sm, lc, cache.block_size, rot, self.final_norm if i == last else None)
            if keep is not None:
                keep.append(x.clone())
        self.last_hidden = x
        return h

    def compute_logits(self, h: torch.Tensor) -> torch.Tensor:
        return F.linear(h, self.embed)

    def set_moe_comm(self, mode: str):
        pass


def count_params(cfg: ModelConfig) -> int:
    W = cfg.hidden_size
    n = cfg.vocab_size * W + 2 * W
    for spec in cfg.layer_specs:
        m = spec["mixer"]
        n += W
        if spec["type"] == "retention":
            n += (2 * m["heads"] * m["dim"] + 3 * m["heads"] * m["vdim"]) * W
        else:
            a, r = m["left"], m["right"]
            nq, nk, nv = a["heads"] * a["dim"], a["kv_heads"] * a["dim"], a["kv_heads"] * a["vdim"]
            n += (nq + nk + nv + a["heads"]) * W + nq + nk + W * a["heads"] * a["vdim"]
            rn, rk = r["heads"] * r["dim"], r.get("decay_rank", 16)
            n += 5 * W + 5 * rn * W + rk * W + rn * rk + 3 * rn
        mlp = spec.get("mlp")
        if mlp is not None:
            n += W
            if mlp["kind"] == "dense":
                n += 3 * W * mlp["ff"]
            else:
                E = mlp["router"]["experts"]
                n += E * W + E + 3 * E * W * mlp["expert"]["ff"]
    return n
