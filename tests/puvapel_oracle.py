"""Plain, slow implementation of the Puvapel design for the tests.

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


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + z.clamp(min=0)


def silu(z):
    return z * sigmoid(z)


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit_length(x, eps=1e-6):
    """x / sqrt(sum(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + eps)


def offset_norm(x, w, eps):
    """RMS norm whose weight is stored around zero."""
    return unit_rms(x, eps) * (1.0 + _f(w))


def cap_of(z, cap):
    return cap * torch.tanh(z / cap) if cap else z


# ---------------------------------------------------------- convolution
def causal_conv(x, w, b=None):
    """Per-channel convolution over time; w[:, -1] meets the current
    token, zeros stand before the start."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            src = t - (taps - 1) + j
            if src >= 0:
                out[t] = out[t] + w[:, j] * x[src]
        if b is not None:
            out[t] = out[t] + b
    return out


# ------------------------------------------------------------ delta rule
def channel_delta(W, p, m, h, eps):
    """Gated delta rule with one decay per head and key channel; several
    heads may share a query/key head."""
    T = h.shape[0]
    H, G, D, Dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), \
        int(m["vdim"])

    def branch(name):
        return silu(causal_conv(h @ _f(W[p + name]).t(),
                                _f(W[p + name + ".conv"])))
    q = unit_length(branch("q").view(T, G, D)) * D ** -0.5
    k = unit_length(branch("k").view(T, G, D))
    v = branch("v").view(T, H, Dv)
    beta = sigmoid(h @ _f(W[p + "b"]).t())                      # (T, H)
    z = ((h @ _f(W[p + "a1"]).t()) @ _f(W[p + "a2"]).t()
         + _f(W[p + "dt_bias"])).view(T, H, D)
    g = torch.exp(-torch.exp(_f(W[p + "A_log"])).view(1, H, 1) * softplus(z))
    gate = sigmoid((h @ _f(W[p + "g1"]).t()) @ _f(W[p + "g2"]).t()
                   ).view(T, H, Dv)
    out = torch.zeros(T, H, Dv, dtype=DT)
    for a in range(H):
        S = torch.zeros(D, Dv, dtype=DT)
        c = a // (H // G)
        for t in range(T):
            S = g[t, a].unsqueeze(1) * S
            u = beta[t, a] * (v[t, a] - S.t() @ k[t, c])
            S = S + torch.outer(k[t, c], u)
            out[t, a] = S.t() @ q[t, c]
    y = unit_rms(out, eps) * _f(W[p + "norm"]) * gate
    return y.reshape(T, H * Dv) @ _f(W[p + "o"]).t()


# ------------------------------------------------------------- attention
def turn(vec, pos, dims, base):
    """Rotate the first ``dims`` entries: pairs (i, i + dims/2)."""
    out = vec.clone()
    half = dims // 2
    for i in range(half):
        a = pos * base ** (-2.0 * i / dims)
        c, s = math.cos(a), math.sin(a)
        out[i] = vec[i] * c - vec[i + half] * s
        out[i + half] = vec[i + half] * c + vec[i] * s
    return out


def chunked_attention(W, p, m, h, eps):
    """Grouped-query attention inside chunks of positions; one is added to
    the softmax denominator."""
    T = h.shape[0]
    H, G, D, Dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), \
        int(m["vdim"])
    size, cap = int(m["mask"]["size"]), float(m.get("softcap") or 0.0)
    rot = m.get("rot") or {}
    dims, base = int(rot.get("dims", 0)), float(rot.get("base", 1e4))

    def branch(name, n, d):
        return causal_conv(h @ _f(W[p + name]).t(),
                           _f(W[p + name + ".conv"])).view(T, n, d)
    q = unit_rms(branch("q", H, D), eps) * _f(W[p + "q.norm"])
    k = unit_rms(branch("k", G, D), eps) * _f(W[p + "k.norm"])
    v = branch("v", G, Dv)
    for t in range(T):
        for a in range(H):
            q[t, a] = turn(q[t, a], t, dims, base)
        for a in range(G):
            k[t, a] = turn(k[t, a], t, dims, base)
    out = torch.zeros(T, H * Dv, dtype=DT)
    for i in range(T):
        j0 = i // size * size                       # first key of the chunk
        for a in range(H):
            c = a // (H // G)
            s = cap_of((k[j0:i + 1, c] @ q[i, a]) * float(m["scale"]), cap)
            e = torch.exp(s)
            w = e / (1.0 + e.sum())
            out[i, a * Dv:(a + 1) * Dv] = w @ v[j0:i + 1, c]
    return out @ _f(W[p + "o"]).t()


# -------------------------------------------------------- selective scan
def selective_scan(W, p, m, h):
    T = h.shape[0]
    C, N, R = int(m["inner"]), int(m["state"]), int(m["dt_rank"])
    xz = h @ _f(W[p + "in"]).t()
    x = silu(causal_conv(xz[:, :C], _f(W[p + "conv"]), _f(W[p + "conv.b"])))
    z = xz[:, C:]
    dbc = x @ _f(W[p + "x"]).t()
    dt = softplus(dbc[:, :R] @ _f(W[p + "dt"]).t() + _f(W[p + "dt.b"]))
    B, Cm = dbc[:, R:R + N], dbc[:, R + N:]
    A = -torch.exp(_f(W[p + "A_log"]))
    S = torch.zeros(C, N, dtype=DT)
    y = torch.zeros(T, C, dtype=DT)
    for t in range(T):
        S = torch.exp(dt[t].unsqueeze(1) * A) * S + \
            torch.outer(dt[t] * x[t], B[t])
        y[t] = S @ Cm[t] + _f(W[p + "D"]) * x[t]
    return (y * silu(z)) @ _f(W[p + "o"]).t()


def parallel(W, p, m, h, eps):
    return float(m["left_scale"]) * \
        chunked_attention(W, p + "left.", m["left"], h, eps) + \
        float(m["right_scale"]) * \
        selective_scan(W, p + "right.", m["right"], h)


# ---------------------------------------------------------- feed-forward
def gated_ff(W, p, h):
    return (silu(h @ _f(W[p + "gate"]).t()) * (h @ _f(W[p + "up"]).t())) \
        @ _f(W[p + "down"]).t()


# ----------------------------------------------------------------- model
def layer(W, li, L, x, eps):
    """Both sublayers read the stream itself; the norm stands on what a
    sublayer gives back."""
    p = f"l{li}."
    mix = channel_delta if L["type"] == "channel_delta" else parallel
    x = x + offset_norm(mix(W, p + "mix.", L["mixer"], x, eps),
                        W[p + "norm1"], eps)
    if L.get("mlp") is not None:
        x = x + offset_norm(gated_ff(W, p + "mlp.", x), W[p + "norm2"], eps)
    return x


def forward(cfg, W, tokens, collect=None):
    """Logits [T, vocab] of one whole sequence; ``collect`` gathers the
    stream after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = _f(W["embed"])[torch.tensor(tokens)]
    for li, L in enumerate(cfg["layers"]):
        x = layer(W, li, L, x, eps)
        if collect is not None:
            collect.append(x.clone())
    return cap_of(offset_norm(x, W["final.norm"], eps) @ _f(W["head"]).t(),
                  float(cfg.get("logit_softcap") or 0.0))


# --------------------------------------------------------------- weights
def random_weights(cfg, seed=0, decay_rank=5, gate_rank=7):
    """name -> tensor for a config; values are bf16-representable so every
    engine dtype loads them exactly."""
    g = torch.Generator().manual_seed(seed)
    Wd, V = int(cfg["width"]), int(cfg["vocab"])

    def rnd(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean) \
            .bfloat16().float()

    def lin(o, i, gain=1.0):
        return rnd(o, i, std=gain / math.sqrt(i))
    W = {"embed": rnd(V, Wd), "final.norm": rnd(Wd, std=0.1),
         "head": lin(V, Wd)}
    for li, L in enumerate(cfg["layers"]):
        p, m = f"l{li}.", L["mixer"]
        q = p + "mix."
        W[p + "norm1"] = rnd(Wd, std=0.2)
        if L["type"] == "channel_delta":
            H, G = int(m["heads"]), int(m["kv_heads"])
            D, Dv, taps = int(m["dim"]), int(m["vdim"]), int(m["conv"])
            for n, rows in (("q", G * D), ("k", G * D), ("v", H * Dv)):
                W[q + n] = lin(rows, Wd)
                W[q + n + ".conv"] = rnd(rows, taps, std=0.6)
            W[q + "b"] = lin(H, Wd, gain=2.0)
            W[q + "A_log"] = rnd(H, std=0.7, mean=-0.5)
            W[q + "norm"] = rnd(Dv, std=0.1, mean=1.0)
            W[q + "a1"], W[q + "a2"] = lin(decay_rank, Wd), \
                lin(H * D, decay_rank)
            W[q + "dt_bias"] = rnd(H * D, mean=-2.0)
            W[q + "g1"], W[q + "g2"] = lin(gate_rank, Wd), \
                lin(H * Dv, gate_rank)
            W[q + "o"] = lin(Wd, H * Dv)
        else:
            a, r = m["left"], m["right"]
            H, G = int(a["heads"]), int(a["kv_heads"])
            D, Dv, taps = int(a["dim"]), int(a["vdim"]), int(a["conv"])
            s = q + "left."
            for n, rows in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                W[s + n] = lin(rows, Wd)
                W[s + n + ".conv"] = rnd(rows, taps, std=0.6)
            W[s + "q.norm"] = rnd(D, std=0.2, mean=1.3)
            W[s + "k.norm"] = rnd(D, std=0.2, mean=1.3)
            W[s + "o"] = lin(Wd, H * Dv)
            s = q + "right."
            C, N, R = int(r["inner"]), int(r["state"]), int(r["dt_rank"])
            W[s + "in"] = lin(2 * C, Wd)
            W[s + "conv"] = rnd(C, int(r["conv"]), std=0.6)
            W[s + "conv.b"] = rnd(C, std=0.2)
            W[s + "x"] = lin(R + 2 * N, C)
            W[s + "dt"], W[s + "dt.b"] = lin(C, R), rnd(C, mean=-1.5)
            W[s + "A_log"] = rnd(C, N, std=0.7)
            W[s + "D"] = rnd(C, std=0.5, mean=1.0)
            W[s + "o"] = lin(Wd, C)
        f = L.get("mlp")
        if f is not None:
            W[p + "norm2"] = rnd(Wd, std=0.2)
            ff = int(f["ff"])
            W[p + "mlp.gate"], W[p + "mlp.up"] = lin(ff, Wd), lin(ff, Wd)
            W[p + "mlp.down"] = lin(Wd, ff)
    return W
