"""A plain, slow float64 model of the Noridra design: one function per
mechanism, whole sequences only (no cache, no state, no batching), written
from the equations and sharing no code with the package.

Notation: x [T, W] is the residual stream for positions 0 .. T-1 of one
sequence, h a sublayer's input, `t` the dict of checkpoint tensors (float64),
`p` a tensor-name prefix, `m` the part of config.json that describes the
mechanism.
"""
import math

import torch

F64 = torch.float64


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + z.clamp_min(0)


def lin(x, w):
    return x @ w.T


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


# ---- embedding, norm, input convolution, output -----------------------------
def embed(tokens, t):
    ids = torch.as_tensor(tokens, dtype=torch.long)
    x = t["embed"][ids]
    if "pos" in t:
        x = x + t["pos"][: len(tokens)]
    return x


def group_norm(x, w, cfg):
    """RMS norm of each of `groups` equal runs of neighbouring entries."""
    n = cfg["norm"]
    G = int(n.get("groups") or 1)
    parts = x.reshape(x.shape[0], G, -1)
    return unit_rms(parts, float(n["eps"])).reshape(x.shape) * w


def short_conv(u, w):
    """y[i] = sum_j w[:, j] u[i - taps + 1 + j], zeros before row 0.
    u [T, C], w [C, taps]."""
    T, C = u.shape
    taps = w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, C, dtype=F64), u], 0)
    y = torch.zeros(T, C, dtype=F64)
    for j in range(taps):
        y = y + w[:, j] * pad[j: j + T]
    return y


def canon(h, w):
    """A sublayer's input: h plus a short convolution of h over time."""
    return h + short_conv(h, w)


def logits(x, t, cfg):
    return lin(group_norm(x, t["final.norm"], cfg), t["head"])


# ---- gated delta rule -------------------------------------------------------
def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_mixer(h, t, p, m, eps):
    T = h.shape[0]
    H, G = int(m["heads"]), int(m["kv_heads"])
    D, V = int(m["dim"]), int(m["vdim"])

    def branch(n):
        u = lin(h, t[p + n])
        return silu(short_conv(u, t[p + n + ".conv"]))

    q = unit(branch("q").view(T, G, D)) * D ** -0.5
    k = unit(branch("k").view(T, G, D))
    v = branch("v").view(T, H, V)
    beta = torch.sigmoid(lin(h, t[p + "b"]))
    g = torch.exp(-torch.exp(t[p + "A_log"]) *
                  softplus(lin(h, t[p + "a"]) + t[p + "dt_bias"]))
    o = torch.zeros(T, H, V, dtype=F64)
    for hd in range(H):
        S = torch.zeros(D, V, dtype=F64)
        kh = hd // (H // G)
        for i in range(T):
            S = g[i, hd] * S
            u = beta[i, hd] * (v[i, hd] - S.T @ k[i, kh])
            S = S + torch.outer(k[i, kh], u)
            o[i, hd] = S.T @ q[i, kh]
    o = unit_rms(o, eps) * t[p + "norm"] * silu(lin(h, t[p + "g"])).view(
        T, H, V)
    return lin(o.reshape(T, H * V), t[p + "o"])


# ---- chunk-local softmax attention, values = keys, sink ---------------------
def attention_mixer(h, t, p, m, eps):
    T = h.shape[0]
    H, G, D = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    size = int(m["mask"]["size"]) if m.get("mask") else 0
    cap = float(m.get("softcap") or 0.0)
    q = unit_rms(lin(h, t[p + "q"]).view(T, H, D), eps) * t[p + "q.norm"]
    v = lin(h, t[p + "k"]).view(T, G, D)
    k = unit_rms(v, eps) * t[p + "k.norm"]
    o = torch.zeros(T, H, D, dtype=F64)
    for hd in range(H):
        g = hd // (H // G)
        for i in range(T):
            lo = i // size * size if size else 0
            s = (k[lo: i + 1, g] @ q[i, hd]) * float(m["scale"])
            if cap:
                s = cap * torch.tanh(s / cap)
            dist = (i - torch.arange(lo, i + 1)).to(F64)
            s = s - t[p + "r1"][hd] * torch.log1p(t[p + "r2"][hd] * dist)
            top = max(float(s.max()), 0.0)
            e = torch.exp(s - top)
            w = e / (math.exp(-top) + e.sum())
            o[i, hd] = w @ v[lo: i + 1, g]
    o = o.reshape(T, H * D) * torch.sigmoid(lin(h, t[p + "g"]))
    return lin(o, t[p + "o"])


# ---- selective scan ---------------------------------------------------------
def mamba_mixer(h, t, p, m, eps=None):
    T = h.shape[0]
    I, N, R = int(m["inner"]), int(m["state"]), int(m["dt_rank"])
    xz = lin(h, t[p + "in"])
    x, z = xz[:, :I], xz[:, I:]
    x = silu(short_conv(x, t[p + "conv"]) + t[p + "conv.b"])
    dbc = lin(x, t[p + "x"])
    dt = softplus(lin(dbc[:, :R], t[p + "dt"]) + t[p + "dt.b"])
    B, C = dbc[:, R: R + N], dbc[:, R + N:]
    A = -torch.exp(t[p + "A_log"])
    S = torch.zeros(I, N, dtype=F64)
    y = torch.zeros(T, I, dtype=F64)
    for i in range(T):
        S = torch.exp(dt[i][:, None] * A) * S + \
            (dt[i] * x[i])[:, None] * B[i][None]
        y[i] = S @ C[i] + t[p + "D"] * x[i]
    return lin(y * silu(z), t[p + "o"])


MIXERS = {"delta": delta_mixer, "attention": attention_mixer,
          "mamba1": mamba_mixer}


# ---- mixture of experts -----------------------------------------------------
def route(h, t, p, r, given=None):
    """-> (chosen experts [T, top], their weights [T, top]). `given` is a
    choice made elsewhere on rounded numbers: it is taken over where its
    scores are within a small distance of the best ones (a close call), so
    that both sides go on with the same experts."""
    top = int(r["top"])
    s = torch.sigmoid(lin(h, t[p + "router"]))
    pick = torch.sort(s, dim=-1, descending=True,
                      stable=True).indices[:, :top]
    if given is not None:
        assert all(len(set(row.tolist())) == top for row in given)
        best, theirs = s.gather(1, pick), s.gather(1, given)
        close = (best.min(-1).values - theirs.min(-1).values) < 0.1
        pick = torch.where(close[:, None], given, pick)
    return pick, s.gather(1, pick)


def expert(h, t, p):
    return lin(silu(lin(h, t[p + "gate"])) * lin(h, t[p + "up"]),
               t[p + "down"])


def moe(h, t, p, f, given=None):
    pick, w = route(h, t, p, f["router"], given)
    out = torch.zeros_like(h)
    for i in range(h.shape[0]):
        for e, we in zip(pick[i].tolist(), w[i]):
            out[i] += expert(we * h[i: i + 1], t, p + f"e{e}.")[0]
    return out


# ---- the whole model --------------------------------------------------------
def forward(tokens, tensors, cfg, taps=None, choices=None):
    """-> logits [T, vocab]; `taps`, if a list, receives the residual stream
    after every layer. `choices`: per layer with a feed-forward, experts
    chosen elsewhere [T, top] (see route)."""
    choices = list(choices) if choices is not None else None
    t = {k: v.to(F64) for k, v in tensors.items()}
    eps = float(cfg["norm"]["eps"])
    alpha = float(cfg["postln_alpha"])
    x = embed(tokens, t)
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = MIXERS[L["type"]](canon(x, t[p + "canon1"]), t, p + "mix.",
                              L["mixer"], eps)
        x = group_norm(alpha * x + t[p + "ls1"] * y, t[p + "norm1"], cfg)
        if L.get("mlp"):
            y = moe(canon(x, t[p + "canon2"]), t, p + "mlp.", L["mlp"],
                    choices.pop(0) if choices is not None else None)
            x = group_norm(alpha * x + t[p + "ls2"] * y, t[p + "norm2"], cfg)
        if taps is not None:
            taps.append(x)
    return logits(x, t, cfg)
