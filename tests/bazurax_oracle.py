"""Dense fp64 forms of every Bazurax mechanism, one function per mechanism, for whole sequences at once.

Written from the design's equations; shares no code with xgserve. `weights` maps checkpoint tensor names to tensors,
`cfg` is the checkpoint's configuration dictionary. Everything is O(T^2) / token-by-token and meant for short inputs.
"""
import math

import torch

F64 = torch.float64


def d(t):
    return t.to(F64)


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, eps):
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def rotate_half(x, pos, rot):
    """x [T, heads, dim]; entries i and i + n / 2 of each head's first n = rot.dims turn by pos * base^(-2 i / n)."""
    n = int(rot["dims"]) if rot else 0
    if n == 0:
        return x
    f = torch.tensor([float(rot["base"]) ** (-2.0 * i / n) for i in range(n // 2)], dtype=F64)
    ang = pos.to(F64)[:, None] * f[None, :]
    c, s = ang.cos()[:, None, :], ang.sin()[:, None, :]
    u, v = x[..., :n // 2], x[..., n // 2:n]
    out = x.clone()
    out[..., :n // 2] = u * c - v * s
    out[..., n // 2:n] = v * c + u * s
    return out


def retention_core(q, k, v, decay, S=None):
    """q, k [T, H, dk], v [T, H, dv], decay [H]: S <- decay_h S + k v^T, o = S^T q. Returns (o [T, H, dv], last S)."""
    T, H, dk = q.shape
    S = torch.zeros(H, dk, v.shape[-1], dtype=F64) if S is None else S.clone()
    rows = []
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        rows.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(rows), S


def retention(h, w, pre, m, eps):
    T = h.shape[0]
    H, dk, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    pos = torch.arange(T)
    q = rotate_half((h @ d(w[pre + "q"]).T).reshape(T, H, dk), pos, m.get("rot"))
    k = rotate_half((h @ d(w[pre + "k"]).T).reshape(T, H, dk), pos, m.get("rot")) * dk ** -0.5
    v = (h @ d(w[pre + "v"]).T).reshape(T, H, dv)
    o, _ = retention_core(q, k, v, torch.tensor([float(a) for a in m["decay"]], dtype=F64))
    y = unit_rms(o, eps).reshape(T, H * dv) * silu(h @ d(w[pre + "g"]).T)
    return y @ d(w[pre + "o"]).T


def window_attention(h, w, pre, m, eps):
    """Sliding-window softmax attention without positions; q / k normed over their whole rows; one gate per head."""
    T = h.shape[0]
    H, G, dk, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = (unit_rms(h @ d(w[pre + "q"]).T, eps) * d(w[pre + "q.norm"])).reshape(T, H, dk)
    k = (unit_rms(h @ d(w[pre + "k"]).T, eps) * d(w[pre + "k.norm"])).reshape(T, G, dk)
    v = (h @ d(w[pre + "v"]).T).reshape(T, G, dv)
    size = int(m["mask"]["size"])
    out = torch.zeros(T, H, dv, dtype=F64)
    for i in range(T):
        lo = max(0, i - size + 1)
        for hh in range(H):
            c = hh // (H // G)
            p = torch.softmax((k[lo:i + 1, c] @ q[i, hh]) * float(m["scale"]), 0)
            out[i, hh] = p @ v[lo:i + 1, c]
    gate = torch.sigmoid(h @ d(w[pre + "g"]).T)
    return (out * gate[:, :, None]).reshape(T, H * dv) @ d(w[pre + "o"]).T


def bonus_core(r, k, v, dec, u, S=None):
    """r, k, v, dec [T, H, D], u [H, D]: o = (S + diag(u) k v^T)^T r, then S <- diag(dec) S + k v^T."""
    T, H, D = r.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=F64) if S is None else S.clone()
    rows = []
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        rows.append(((S + u[:, :, None] * kv) * r[t][:, :, None]).sum(1))
        S = dec[t][:, :, None] * S + kv
    return torch.stack(rows), S


def token_shift(h, mu, prev=None):
    """h + (h' - h) mu, h' the previous token's row (zeros, or `prev`, before the first)."""
    first = torch.zeros(1, h.shape[1], dtype=F64) if prev is None else prev.reshape(1, -1)
    return h + (torch.cat([first, h[:-1]]) - h) * mu


def time_mix(h, w, pre, m, eps):
    T = h.shape[0]
    H, D = int(m["heads"]), int(m["dim"])
    mixed = {s: token_shift(h, d(w[pre + "mu." + s])) for s in "rkvgw"}
    r, k, v = ((mixed[s] @ d(w[pre + s]).T).reshape(T, H, D) for s in "rkv")
    gate = silu(mixed["g"] @ d(w[pre + "g"]).T)
    z = torch.tanh(mixed["w"] @ d(w[pre + "w1"]).T) @ d(w[pre + "w2"]).T + d(w[pre + "w0"])
    dec = torch.exp(-torch.exp(z)).reshape(T, H, D)
    o, _ = bonus_core(r, k, v, dec, d(w[pre + "u"]).reshape(H, D))
    y = unit_rms(o, eps).reshape(T, H * D) * d(w[pre + "norm"]) * gate
    return y @ d(w[pre + "o"]).T


def parallel_mixer(h, w, pre, m, eps):
    return float(m["left_scale"]) * window_attention(h, w, pre + "left.", m["left"], eps) + \
        float(m["right_scale"]) * time_mix(h, w, pre + "right.", m["right"], eps)


def glu(h, w, pre):
    return (silu(h @ d(w[pre + "gate"]).T) * (h @ d(w[pre + "up"]).T)) @ d(w[pre + "down"]).T


def moe(h, w, pre, mlp):
    """Router logits with a bias; the `top` largest, weighted by the softmax over the chosen logits alone."""
    E, top = int(mlp["router"]["experts"]), int(mlp["router"]["top"])
    z = h @ d(w[pre + "router"]).T + d(w[pre + "router.b"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        order = sorted(range(E), key=lambda e: (-float(z[t, e]), e))[:top]
        p = torch.softmax(z[t, order], 0)
        for j, e in enumerate(order):
            out[t] += p[j] * glu(h[t:t + 1], w, f"{pre}e{e}.")[0]
    return out


def forward(cfg, w, tokens, keep=None):
    """Logits [T, vocab] of one whole sequence; `keep` collects the residual stream after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = layer_norm(d(w["embed"])[torch.as_tensor(tokens).long()], d(w["embed.norm"]), eps)
    for i, L in enumerate(cfg["layers"]):
        pre = f"l{i}."
        f = retention if L["type"] == "retention" else parallel_mixer
        x = x + layer_norm(f(x, w, pre + "mix.", L["mixer"], eps), d(w[pre + "norm1"]), eps)
        mlp = L.get("mlp")
        if mlp is not None:
            y = glu(x, w, pre + "mlp.") if mlp["kind"] == "dense" else moe(x, w, pre + "mlp.", mlp)
            x = x + layer_norm(y, d(w[pre + "norm2"]), eps)
        if keep is not None:
            keep.append(x.clone())
    return layer_norm(x, d(w["final.norm"]), eps) @ d(w["embed"]).T


def random_weights(cfg, seed=0):
    """Random weights of a configuration, rounded to bfloat16 (what a checkpoint stores). Recurrent queries and keys are
    correlated (and the bonus is mostly positive), so that a token's own key scores clearly above zero: an output whose terms
    almost cancel is blown up by its head norm, rounding included, and early tokens have few terms. `decay_rank` of a right branch
    (the rank of its decay projection) is read from the mixer's dictionary and not written to config.json."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    out = {}

    def mat(name, o, i, gain=1.0):
        out[name] = torch.randn(o, i, generator=g) * gain / math.sqrt(i)

    def vec(name, n, std, mean=0.0):
        out[name] = torch.randn(n, generator=g) * std + mean
    out["embed"] = torch.randn(V, W, generator=g) * 0.5
    vec("embed.norm", W, 0.2, 1.0)
    vec("final.norm", W, 0.2, 1.0)
    for n, L in enumerate(cfg["layers"]):
        pre, m = f"l{n}.", L["mixer"]
        vec(pre + "norm1", W, 0.2, 0.7)
        if L["type"] == "retention":
            H, dk, dv = m["heads"], m["dim"], m["vdim"]
            for nm, rows in (("q", H * dk), ("k", H * dk), ("v", H * dv), ("g", H * dv)):
                mat(pre + "mix." + nm, rows, W)
            out[pre + "mix.k"] = 0.6 * out[pre + "mix.k"] + 0.8 * out[pre + "mix.q"]
            mat(pre + "mix.o", W, H * dv)
        else:
            a, r = m["left"], m["right"]
            H, G, dk, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            for nm, rows in (("q", H * dk), ("k", G * dk), ("v", G * dv), ("g", H)):
                mat(pre + "mix.left." + nm, rows, W)
            vec(pre + "mix.left.q.norm", H * dk, 0.3, 1.2)
            vec(pre + "mix.left.k.norm", G * dk, 0.3, 1.2)
            mat(pre + "mix.left.o", W, H * dv)
            R, rk = r["heads"] * r["dim"], r.get("decay_rank", 4)
            for s in "rkvgw":
                out[pre + "mix.right.mu." + s] = torch.rand(W, generator=g)
            for s in "rkvg":
                mat(pre + "mix.right." + s, R, W)
            out[pre + "mix.right.k"] = 0.6 * out[pre + "mix.right.k"] + 0.8 * out[pre + "mix.right.r"]
            mat(pre + "mix.right.w1", rk, W)
            mat(pre + "mix.right.w2", R, rk)
            out[pre + "mix.right.w0"] = torch.rand(R, generator=g) * 5.0 - 5.0
            out[pre + "mix.right.u"] = torch.randn(r["heads"], r["dim"], generator=g) * 0.5 + 1.0
            vec(pre + "mix.right.norm", R, 0.3, 1.0)
            mat(pre + "mix.right.o", W, R)
        mlp = L.get("mlp")
        if mlp is None:
            continue
        vec(pre + "norm2", W, 0.2, 0.7)

        def ff(p, n):
            mat(p + "gate", n, W)
            mat(p + "up", n, W)
            mat(p + "down", W, n)
        if mlp["kind"] == "dense":
            ff(pre + "mlp.", mlp["ff"])
        else:
            E = mlp["router"]["experts"]
            mat(pre + "mlp.router", E, W, 2.0)
            vec(pre + "mlp.router.b", E, 0.5)
            for e in range(E):
                ff(f"{pre}mlp.e{e}.", mlp["expert"]["ff"])
    return {k: v.to(torch.bfloat16).to(F64) for k, v in out.items()}


def write_checkpoint(path, cfg, Wt):
    """config.json + model.safetensors (bfloat16) of a test model."""
    import copy
    import json
    import os

    from safetensors.torch import save_file
    c = copy.deepcopy(cfg)
    for L in c["layers"]:
        if L["type"] == "parallel":
            L["mixer"]["right"].pop("decay_rank", None)
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(c, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in Wt.items()}, os.path.join(path, "model.safetensors"))
