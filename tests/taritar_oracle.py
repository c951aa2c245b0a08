"""Dense fp64 forms of every Taritar mechanism, one function per mechanism, for whole sequences at once.

Written from the design's equations; shares no code with xgserve. `weights` maps checkpoint tensor names to tensors,
`cfg` is the checkpoint's configuration dictionary. Everything is O(T^2) / token-by-token and meant for short inputs.
"""
import math

import torch

F64 = torch.float64


def d(t):
    return t.to(F64)


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def embed(cfg, w, tokens):
    """Scaled token rows plus the (unscaled) learned vector of each position."""
    n = len(tokens)
    return d(w["embed"])[torch.as_tensor(tokens).long()] * float(cfg["embedding"]["scale"]) + d(w["pos"])[:n]


# ---------------------------------------------------------------------------------- residual streams
def streams_read(X, w_in):
    """X [S, T, W]: what a sublayer reads, the weighted sum of the streams."""
    return sum(w_in[s] * X[s] for s in range(X.shape[0]))


def streams_write(X, mix, w_out, y):
    """Every new stream t from all old ones: sum_s mix[s, t] X_s + w_out[t] y."""
    S = X.shape[0]
    return torch.stack([sum(mix[s, t] * X[s] for s in range(S)) + w_out[t] * y for t in range(S)])


# ---------------------------------------------------------------------------------- attention
def rotate(x, pos, rot):
    """x [T, heads, dim]: entries 2 i and 2 i + 1 of the first rot.dims turn by pos * base^(-2 i / dims)."""
    n = int(rot["dims"]) if rot else 0
    if n == 0:
        return x
    out = x.clone()
    for i in range(n // 2):
        a = pos.to(F64) * float(rot["base"]) ** (-2.0 * i / n)
        c, s = a.cos()[:, None], a.sin()[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def visible(i, mask):
    """Positions a query at `i` sees: a sliding window ending at it, and the sequence's first tokens."""
    if not mask:
        return list(range(i + 1))
    return [j for j in range(i + 1) if i - j < int(mask["size"]) or j < int(mask.get("keep_first", 0))]


def keys_values(h, w, pre, m):
    """(rotated keys [T, G, dim], values [T, G, vdim]) of a layer with projections of its own."""
    T, G = h.shape[0], int(m["kv_heads"])
    k = (h @ d(w[pre + "k"]).T).reshape(T, G, int(m["dim"]))
    v = (h @ d(w[pre + "v"]).T).reshape(T, G, int(m["vdim"]))
    return rotate(k, torch.arange(T), m.get("rot")), v


def attend(q, k, v, m):
    """q [T, H, dim] rotated; capped scores over the visible keys, softmax, weighted values [T, H, vdim]."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=F64)
    cap = m.get("softcap")
    for i in range(T):
        vis = visible(i, m.get("mask"))
        for h in range(H):
            g = h // (H // G)
            sc = (k[vis, g] @ q[i, h]) * float(m["scale"])
            if cap:
                sc = float(cap) * torch.tanh(sc / float(cap))
            out[i, h] = torch.softmax(sc, 0) @ v[vis, g]
    return out


def attention(h, w, pre, m, kv):
    T, H = h.shape[0], int(m["heads"])
    q = rotate((h @ d(w[pre + "q"]).T).reshape(T, H, int(m["dim"])), torch.arange(T), m.get("rot"))
    return attend(q, kv[0], kv[1], m).reshape(T, -1) @ d(w[pre + "o"]).T


# ---------------------------------------------------------------------------------- feed-forward
def clamped_glu(h, w, pre, limit):
    g = torch.clamp(h @ d(w[pre + "gate"]).T, max=limit)
    u = torch.clamp(h @ d(w[pre + "up"]).T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ d(w[pre + "down"]).T


def route(z, router):
    """Router logits of one token [E] -> [(expert, weight)]: softmax scores over all experts; the groups with the largest
    best member are eligible; the largest eligible scores win and are the weights as they are."""
    E = z.shape[0]
    s = torch.softmax(z, 0)
    groups = router.get("groups") or {"count": 1, "keep": 1}
    per = E // int(groups["count"])
    best = [max(float(s[e]) for e in range(g * per, (g + 1) * per)) for g in range(int(groups["count"]))]
    kept = sorted(range(len(best)), key=lambda g: (-best[g], g))[:int(groups["keep"])]
    cand = [e for e in range(E) if e // per in kept]
    return [(e, s[e]) for e in sorted(cand, key=lambda e: (-float(s[e]), e))[:int(router["top"])]]


def moe(h, w, pre, mlp):
    z = h @ d(w[pre + "router"]).T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in route(z[t], mlp["router"]):
            out[t] += s * clamped_glu(h[t:t + 1], w, f"{pre}e{e}.", float(mlp["expert"]["limit"]))[0]
    if mlp.get("shared"):
        y = clamped_glu(h, w, pre + "shared.", float(mlp["shared"]["limit"]))
        out = out + torch.sigmoid(h @ d(w[pre + "shared.sg"]).T) * y
    return out


def soft_cap(x, cap):
    return cap * torch.tanh(x / cap) if cap else x


def forward(cfg, w, tokens, keep=None):
    """Logits [T, vocab] of one whole sequence; `keep` collects the sum of the streams after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = embed(cfg, w, tokens)
    X = torch.stack([x] * int(cfg["streams"]))
    kvs = {}
    for i, L in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", L["mixer"]
        h = rms_norm(streams_read(X, d(w[pre + "hc1.in"])), d(w[pre + "norm1"]), eps)
        if m.get("kv_from") is None:
            kvs[i] = keys_values(h, w, pre + "mix.", m)
        y = attention(h, w, pre + "mix.", m, kvs[i if m.get("kv_from") is None else int(m["kv_from"])])
        X = streams_write(X, d(w[pre + "hc1.mix"]), d(w[pre + "hc1.out"]), y)
        mlp = L.get("mlp")
        if mlp is not None:
            h = rms_norm(streams_read(X, d(w[pre + "hc2.in"])), d(w[pre + "norm2"]), eps)
            y = clamped_glu(h, w, pre + "mlp.", float(mlp["limit"])) if mlp["kind"] == "dense" else moe(h, w, pre + "mlp.", mlp)
            X = streams_write(X, d(w[pre + "hc2.mix"]), d(w[pre + "hc2.out"]), y)
        if keep is not None:
            keep.append(X.sum(0))
    return soft_cap(rms_norm(X.sum(0), d(w["final.norm"]), eps) @ d(w["head"]).T, cfg.get("logit_softcap"))


# ---------------------------------------------------------------------------------- test models
def random_weights(cfg, seed=0):
    """Random weights of a configuration, rounded to bfloat16 (what a checkpoint stores)."""
    g = torch.Generator().manual_seed(seed)
    W, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    out = {}

    def mat(name, o, i, gain=1.0):
        out[name] = torch.randn(o, i, generator=g) * gain / math.sqrt(i)

    def vec(name, n, std, mean=0.0):
        out[name] = torch.randn(n, generator=g) * std + mean

    def glu(pre, ff):
        mat(pre + "gate", ff, W)
        mat(pre + "up", ff, W)
        mat(pre + "down", W, ff)

    def hyper(pre):
        vec(pre + "in", S, 0.3, 1.0 / S)
        vec(pre + "out", S, 0.4, 1.0)
        out[pre + "mix"] = 0.8 * torch.eye(S) + torch.randn(S, S, generator=g) * 0.3 / S
    out["embed"] = torch.randn(V, W, generator=g)
    out["pos"] = torch.randn(cfg["max_positions"], W, generator=g) * 0.3
    mat("head", V, W, 3.0)
    vec("final.norm", W, 0.2, 1.0)
    for n, L in enumerate(cfg["layers"]):
        pre, m, mlp = f"l{n}.", L["mixer"], L.get("mlp")
        H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        vec(pre + "norm1", W, 0.2, 1.0)
        hyper(pre + "hc1.")
        mat(pre + "mix.q", H * dk, W, 1.2)
        if m.get("kv_from") is None:
            mat(pre + "mix.k", G * dk, W, 1.2)
            mat(pre + "mix.v", G * dv, W)
        mat(pre + "mix.o", W, H * dv)
        if mlp is None:
            continue
        vec(pre + "norm2", W, 0.2, 1.0)
        hyper(pre + "hc2.")
        if mlp["kind"] == "dense":
            glu(pre + "mlp.", mlp["ff"])
            continue
        mat(pre + "mlp.router", mlp["router"]["experts"], W, 2.0)
        for e in range(mlp["router"]["experts"]):
            glu(f"{pre}mlp.e{e}.", mlp["expert"]["ff"])
        if mlp.get("shared"):
            glu(pre + "mlp.shared.", mlp["shared"]["ff"])
            mat(pre + "mlp.shared.sg", 1, W, 2.0)
    return {k: v.to(torch.bfloat16).to(F64) for k, v in out.items()}


def write_checkpoint(path, cfg, weights):
    """config.json + model.safetensors (bfloat16) of a test model."""
    import json
    import os

    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in weights.items()}, os.path.join(path, "model.safetensors"))
