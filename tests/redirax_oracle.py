"""Plain, slow implementation of the Redirax design for the tests.

One function per mechanism, written from the design's equations; whole
sequences only (no cache, no batching, no paging, no recurrent state that
outlives a call).  It shares no code with ``polyrl_amd``: the engine, its
cache manager and its kernels are compared against these functions.

Conventions: ``W`` maps tensor names to torch tensors, linear weights are
[out, in] and applied as ``W @ x``; ``cfg`` is the parsed config dict.
Everything runs in ``DT`` (float64 by default).
"""
import math

import torch

DT = torch.float64


def _f(t):
    return t.to(DT)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def linear(W, name, x):
    y = x @ _f(W[name]).t()
    return y + _f(W[name + ".b"]) if name + ".b" in W else y


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * _f(w)


def tanh_norm(W, name, x):
    """tanh(alpha x) w + b."""
    return torch.tanh(_f(W[name + ".alpha"]) * x) * _f(W[name]) \
        + _f(W[name + ".b"])


def cap_of(z, cap):
    return cap * torch.tanh(z / cap) if cap else z


# ------------------------------------------------------ softmax attention
def pair_angles(T, rot):
    """(T, dims/2) angles p * base^(-2i/dims) / factor."""
    dims = int(rot["dims"])
    factor = float((rot.get("scaling") or {}).get("factor", 1.0))
    f = torch.tensor([float(rot["base"]) ** (-2.0 * i / dims) / factor
                      for i in range(dims // 2)], dtype=DT)
    return torch.arange(T, dtype=DT).unsqueeze(1) * f


def rotate_pairs(x, rot):
    """x (T, heads, D): neighbours (2i, 2i + 1) of the first dims entries
    turn by their angle."""
    out = x.clone()
    ang = pair_angles(x.shape[0], rot)
    for i in range(int(rot["dims"]) // 2):
        c, s = torch.cos(ang[:, i:i + 1]), torch.sin(ang[:, i:i + 1])
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i] = u * c - v * s
        out[:, :, 2 * i + 1] = v * c + u * s
    return out


def attention(W, p, a, h):
    """Causal grouped-query softmax attention with projection biases."""
    T = h.shape[0]
    H, G, D, Dv = (int(a[n]) for n in ("heads", "kv_heads", "dim", "vdim"))
    q = linear(W, p + "q", h).view(T, H, D)
    k = linear(W, p + "k", h).view(T, G, D)
    v = linear(W, p + "v", h).view(T, G, Dv)
    rot = a.get("rot")
    if rot and int(rot["dims"]):
        q, k = rotate_pairs(q, rot), rotate_pairs(k, rot)
    seen = torch.ones(T, T, dtype=torch.bool).tril()
    out = torch.zeros(T, H, Dv, dtype=DT)
    for n in range(H):
        g = n // (H // G)
        s = (q[:, n] @ k[:, g].t()) * float(a["scale"])
        s = s.masked_fill(~seen, -math.inf)
        e = torch.exp(s - s.max(-1, keepdim=True).values)
        out[:, n] = (e / e.sum(-1, keepdim=True)) @ v[:, g]
    return linear(W, p + "o", out.reshape(T, H * Dv))


# ---------------------------------------------------- lightning attention
def lightning(W, p, r, h, eps):
    """S <- decay S + k v^T, o = S^T q per head, one token after the other;
    the row of all heads is normed and gated."""
    T = h.shape[0]
    H, D, Dv = int(r["heads"]), int(r["dim"]), int(r["vdim"])
    q = silu(linear(W, p + "q", h)).view(T, H, D)
    k = silu(linear(W, p + "k", h)).view(T, H, D)
    v = silu(linear(W, p + "v", h)).view(T, H, Dv)
    out = torch.zeros(T, H, Dv, dtype=DT)
    for n in range(H):
        S = torch.zeros(D, Dv, dtype=DT)
        for t in range(T):
            S = float(r["decay"][n]) * S + torch.outer(k[t, n], v[t, n])
            out[t, n] = q[t, n] @ S
    y = rms_norm(out.reshape(T, H * Dv), W[p + "norm"], eps)
    return linear(W, p + "o", y * sigmoid(linear(W, p + "g", h)))


def side_by_side(W, p, m, h, eps):
    """Half the sum of the two mixers' normed outputs."""
    left = rms_norm(attention(W, p + "left.", m["left"], h),
                    W[p + "left.out"], eps)
    right = rms_norm(lightning(W, p + "right.", m["right"], h, eps),
                     W[p + "right.out"], eps)
    return (left + right) / 2


# ------------------------------------------------------------ feed-forward
def dense(W, p, f, h):
    gate = linear(W, p + "gate", h)
    return linear(W, p + "down", gate.clamp(min=0) * linear(W, p + "up", h))


def expert(W, p, limit, h):
    g = linear(W, p + "gate", h).clamp(max=limit)
    u = linear(W, p + "up", h).clamp(-limit, limit)
    return linear(W, p + "down", g * sigmoid(1.702 * g) * (u + 1.0))


def router(W, p, top, h):
    """Per token: the experts with the largest logits and the softmax over
    just those logits."""
    z = linear(W, p + "router", h)
    best, idx = z.topk(top, -1)
    e = torch.exp(best - best.max(-1, keepdim=True).values)
    return idx, e / e.sum(-1, keepdim=True)


def experts(W, p, f, h):
    idx, w = router(W, p, int(f["router"]["top"]), h)
    limit = float(f["expert"]["limit"])
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, we in zip(idx[t].tolist(), w[t]):
            y[t] += we * expert(W, f"{p}e{e}.", limit, h[t])
    if f.get("shared"):
        y = y + sigmoid(linear(W, p + "shared.sg", h)) * \
            expert(W, p + "shared.", float(f["shared"]["limit"]), h)
    return y


# --------------------------------------------------------------- the stack
def through_streams(W, p, xs, sublayer):
    """xs (S, T, width): read one mixture of the streams, write the result
    back to all of them, mixed anew."""
    u = torch.einsum("s,stw->tw", _f(W[p + "in"]), xs)
    y = sublayer(u)
    return torch.einsum("st,snw->tnw", _f(W[p + "mix"]), xs) \
        + _f(W[p + "out"])[:, None, None] * y


def forward(cfg, W, tokens, collect=None):
    """Logits (T, vocab) of a whole sequence; ``collect`` receives the sum
    of the streams after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = _f(W["embed"])[torch.as_tensor(tokens)]
    xs = x.unsqueeze(0).repeat(int(cfg["streams"]), 1, 1)
    for li, L in enumerate(cfg["layers"]):
        owner = L.get("weights_of")
        p = f"l{li if owner is None else owner}."
        xs = through_streams(W, p + "hc1.", xs, lambda u: side_by_side(
            W, p + "mix.", L["mixer"], tanh_norm(W, p + "norm1", u), eps))
        f = L.get("mlp")
        if f is not None:
            ff = dense if f["kind"] == "dense" else experts
            xs = through_streams(W, p + "hc2.", xs, lambda u: ff(
                W, p + "mlp.", f, tanh_norm(W, p + "norm2", u)))
        if collect is not None:
            collect.append(xs.sum(0))
    y = tanh_norm(W, "final.norm", xs.sum(0)) @ _f(W["head"]).t()
    return cap_of(y, float(cfg.get("logit_softcap") or 0.0))


# --------------------------------------------------------------- weights
def random_weights(cfg, seed=0):
    """name -> tensor for a config; values are bf16-representable so every
    engine dtype loads them exactly."""
    g = torch.Generator().manual_seed(seed)
    Wd, V, S = int(cfg["width"]), int(cfg["vocab"]), int(cfg["streams"])

    def rnd(*shape, std=1.0, mean=0.0):
        return (torch.randn(shape, generator=g) * std + mean) \
            .bfloat16().float()

    def lin(o, i, gain=1.0):
        return rnd(o, i, std=gain / math.sqrt(i))
    W = {"embed": rnd(V, Wd), "head": lin(V, Wd, gain=2.0)}

    def norm(name):
        W[name] = rnd(Wd, std=0.2, mean=1.0)
        W[name + ".b"] = rnd(Wd, std=0.2)
        W[name + ".alpha"] = rnd(std=0.1, mean=0.7)

    def streams(p):
        W[p + "in"] = rnd(S, std=0.3, mean=1.0 / S)
        W[p + "out"] = rnd(S, std=0.4, mean=1.0)
        W[p + "mix"] = (torch.eye(S) * 0.8
                        + torch.randn(S, S, generator=g) * 0.2) \
            .bfloat16().float()
    norm("final.norm")
    for li, L in enumerate(cfg["layers"]):
        if L.get("weights_of") is not None:
            continue
        p, m = f"l{li}.", L["mixer"]
        norm(p + "norm1")
        streams(p + "hc1.")
        a, q = m["left"], p + "mix.left."
        H, G, D, Dv = (int(a[n]) for n in ("heads", "kv_heads", "dim",
                                           "vdim"))
        for n, rows in (("q", H * D), ("k", G * D), ("v", G * Dv)):
            W[q + n] = lin(rows, Wd)
            W[q + n + ".b"] = rnd(rows, std=0.5)
        W[q + "o"], W[q + "o.b"] = lin(Wd, H * Dv), rnd(Wd, std=0.3)
        W[q + "out"] = rnd(Wd, std=0.2, mean=1.0)
        r, q = m["right"], p + "mix.right."
        H, D, Dv = (int(r[n]) for n in ("heads", "dim", "vdim"))
        for n, rows in (("q", H * D), ("k", H * D), ("v", H * Dv),
                        ("g", H * Dv)):
            W[q + n] = lin(rows, Wd)
        W[q + "norm"] = rnd(H * Dv, std=0.2, mean=1.0)
        W[q + "o"] = lin(Wd, H * Dv)
        W[q + "out"] = rnd(Wd, std=0.2, mean=1.0)
        f = L.get("mlp")
        if f is None:
            continue
        norm(p + "norm2")
        streams(p + "hc2.")
        p += "mlp."

        def glu(q, ff):
            W[q + "gate"], W[q + "up"] = lin(ff, Wd), lin(ff, Wd)
            W[q + "down"] = lin(Wd, ff)
        if f["kind"] == "dense":
            glu(p, int(f["ff"]))
            continue
        E = int(f["router"]["experts"])
        for e in range(E):
            glu(f"{p}e{e}.", int(f["expert"]["ff"]))
        W[p + "router"], W[p + "router.b"] = lin(E, Wd, gain=3.0), \
            rnd(E, std=0.5)
        if f.get("shared"):
            glu(p + "shared.", int(f["shared"]["ff"]))
            W[p + "shared.sg"] = lin(1, Wd)
    return W
