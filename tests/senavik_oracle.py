"""A plain, slow float64 model of the Senavik design: one function per
mechanism, whole sequences only (no cache, no batching), written from the
equations and sharing no code with the package.

Notation: x [T, W] is the residual stream for positions 0 .. T-1 of one
sequence, h a sublayer's input, `t` the dict of checkpoint tensors (float64),
`p` a tensor-name prefix, `m` the part of config.json that describes the
mechanism.
"""
import math

import torch

F64 = torch.float64


def lin(x, w):
    return x @ w.T


def rms(x, eps):
    """x over the root of its mean square."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def offset_norm(x, w, cfg):
    """The stack's own norm: its weight is stored as what it adds to 1."""
    return rms(x, float(cfg["norm"]["eps"])) * (1.0 + w)


def embed(tokens, t, cfg):
    rows = t["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    return offset_norm(rows, t["embed.norm"], cfg)


def logits(x, t, cfg):
    return lin(offset_norm(x, t["final.norm"], cfg), t["head"])


# ---- rotary positions -------------------------------------------------------
def plain_frequency(i, rot):
    return float(rot["base"]) ** (-2.0 * i / int(rot["dims"]))


def banded_frequency(f, s):
    """Short wavelengths keep their frequency, long ones are slowed down by
    the factor, those between the two limits get a blend."""
    wavelength = 2.0 * math.pi / f
    turns = float(s["original"]) / wavelength
    if turns > float(s["high"]):
        return f
    if turns < float(s["low"]):
        return f / float(s["factor"])
    a = (turns - float(s["low"])) / (float(s["high"]) - float(s["low"]))
    return (1.0 - a) * f / float(s["factor"]) + a * f


def ramped_frequency(f, i, rot):
    """The blend runs linearly over the pair index, between the pairs that
    turn `fast` and `slow` times over the original context."""
    s = rot["scaling"]
    dims, base = int(rot["dims"]), float(rot["base"])

    def pair(turns):
        return dims * math.log(float(s["original"]) / (turns * 2.0 * math.pi)
                               ) / (2.0 * math.log(base))
    first = max(math.floor(pair(float(s["fast"]))), 0)
    last = min(math.ceil(pair(float(s["slow"]))), dims - 1)
    r = min(max((i - first) / max(last - first, 0.001), 0.0), 1.0)
    return r * f / float(s["factor"]) + (1.0 - r) * f


def rotation(rot):
    """-> (frequency of every pair, factor of cos and sin)."""
    n = int(rot["dims"]) // 2
    f = [plain_frequency(i, rot) for i in range(n)]
    s = rot.get("scaling")
    if not s:
        return f, 1.0
    if "fast" in s:
        return ([ramped_frequency(f[i], i, rot) for i in range(n)],
                0.1 * math.log(float(s["factor"])) + 1.0)
    return [banded_frequency(fi, s) for fi in f], 1.0


def rotate(x, rot):
    """x [T, heads, D]: entry i < dims/2 turns with entry i + dims/2."""
    T = x.shape[0]
    n = int(rot["dims"]) // 2
    f, amp = rotation(rot)
    y = x.clone()
    for p in range(T):
        for i in range(n):
            c, s = amp * math.cos(p * f[i]), amp * math.sin(p * f[i])
            u, v = x[p, :, i], x[p, :, i + n]
            y[p, :, i] = u * c - v * s
            y[p, :, i + n] = v * c + u * s
    return y


# ---- softmax with a sink ----------------------------------------------------
def sink_weights(s, sink):
    """Weights of scores s [n] when one more score without a value, `sink`,
    takes part (None: none does)."""
    top = float(s.max()) if sink is None else max(float(s.max()), float(sink))
    e = torch.exp(s - top)
    den = e.sum()
    if sink is not None:
        den = den + math.exp(float(sink) - top)
    return e / den


# ---- attention over a window and the first tokens ---------------------------
def visible(i, mask):
    """Positions that position i sees."""
    size = int((mask or {}).get("size") or 0)
    keep = int((mask or {}).get("keep_first") or 0)
    return [j for j in range(i + 1)
            if not size or i - j < size or j < keep]


def attention(h, t, p, m, eps=None):
    T = h.shape[0]
    H, G = int(m["heads"]), int(m["kv_heads"])
    D, V = int(m["dim"]), int(m["vdim"])
    q = rotate(lin(h, t[p + "q"]).view(T, H, D), m["rot"])
    k = rotate(lin(h, t[p + "k"]).view(T, G, D), m["rot"])
    v = lin(h, t[p + "v"]).view(T, G, V)
    o = torch.zeros(T, H, V, dtype=F64)
    for i in range(T):
        js = visible(i, m.get("mask"))
        for hd in range(H):
            g = hd // (H // G)
            w = sink_weights((k[js, g] @ q[i, hd]) * float(m["scale"]),
                             t[p + "sink"][hd])
            o[i, hd] = w @ v[js, g]
    return lin(o.reshape(T, H * V), t[p + "o"])


# ---- latent attention -------------------------------------------------------
def latent_attention(h, t, p, m, eps):
    T = h.shape[0]
    H, D, R = int(m["heads"]), int(m["dim"]), int(m["rot_dim"])
    V, C = int(m["vdim"]), int(m["kv_rank"])
    cq = rms(lin(h, t[p + "dq"]), eps) * t[p + "dq.norm"]
    q = lin(cq, t[p + "uq"]).view(T, H, D + R)
    down = lin(h, t[p + "dkv"])
    c = rms(down[:, :C], eps) * t[p + "dkv.norm"]
    kr = rotate(down[:, C:].view(T, 1, R), m["rot"])[:, 0]
    qr = rotate(q[:, :, D:], m["rot"])
    k = lin(c, t[p + "uk"]).view(T, H, D)
    v = lin(c, t[p + "uv"]).view(T, H, V)
    o = torch.zeros(T, H, V, dtype=F64)
    for i in range(T):
        for hd in range(H):
            s = k[: i + 1, hd] @ q[i, hd, :D] + kr[: i + 1] @ qr[i, hd]
            o[i, hd] = sink_weights(s * float(m["scale"]),
                                    t[p + "sink"][hd]) @ v[: i + 1, hd]
    return lin(o.reshape(T, H * V), t[p + "o"])


MIXERS = {"attention": attention, "latent_attention": latent_attention}


# ---- feed-forward -----------------------------------------------------------
def dense(h, t, p):
    z = lin(h, t[p + "up"]).clamp_min(0.0)
    return lin(z * z, t[p + "down"])


def expert(h, t, p):
    z = lin(h, t[p + "gate"])
    return lin(z * torch.sigmoid(z) * lin(h, t[p + "up"]), t[p + "down"])


def choose(c, top, groups=None):
    """Experts chosen by the choice scores c [E] of one token: the best
    groups by the sum of a group's two largest scores, then the best experts
    of those groups."""
    E = c.shape[0]
    allowed = list(range(E))
    if groups:
        n, keep = int(groups["count"]), int(groups["keep"])
        per = E // n
        value = [sum(sorted(c[g * per: (g + 1) * per].tolist(),
                            reverse=True)[:2]) for g in range(n)]
        best = sorted(range(n), key=lambda g: (-value[g], g))[:keep]
        allowed = [e for e in range(E) if e // per in best]
    return sorted(allowed, key=lambda e: (-float(c[e]), e))[:top]


def route(h, t, p, r, given=None):
    """-> (chosen experts [T, top], their weights [T, top]). `given` is a
    choice made elsewhere on rounded numbers: it is taken over where it
    comes out as the best one after a small change of the scores (a close
    call), so that both sides go on with the same experts."""
    top = int(r["top"])
    s = torch.sigmoid(lin(h, t[p + "router"]))
    c = s + t[p + "correction"]
    pick = torch.tensor([choose(ci, top, r.get("groups")) for ci in c])
    if given is not None:
        assert all(len(set(row.tolist())) == top for row in given)
        lift = torch.zeros_like(c).scatter(1, given, 0.1)
        near = [sorted(choose(ci, top, r.get("groups"))) == sorted(g.tolist())
                for ci, g in zip(c + lift, given)]
        pick = torch.where(torch.tensor(near)[:, None], given, pick)
    w = s.gather(1, pick)
    return pick, w / (w.sum(-1, keepdim=True) + 1e-20)


def moe(h, t, p, f, given=None):
    pick, w = route(h, t, p, f["router"], given)
    out = torch.zeros_like(h)
    for i in range(h.shape[0]):
        for e, we in zip(pick[i].tolist(), w[i]):
            out[i] += we * expert(h[i: i + 1], t, p + f"e{e}.")[0]
    return out


# ---- the whole model --------------------------------------------------------
def forward(tokens, tensors, cfg, taps=None, choices=None):
    """-> logits [T, vocab]; `taps`, if a list, receives the residual stream
    after every layer. `choices`: per layer with experts, experts chosen
    elsewhere [T, top] (see route)."""
    choices = list(choices) if choices is not None else None
    t = {k: v.to(F64) for k, v in tensors.items()}
    eps = float(cfg["norm"]["eps"])
    x = embed(tokens, t, cfg)
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + MIXERS[L["type"]](offset_norm(x, t[p + "norm1"], cfg), t,
                                  p + "mix.", L["mixer"], eps)
        f = L.get("mlp")
        if f:
            h = offset_norm(x, t[p + "norm2"], cfg)
            if f["kind"] == "dense":
                y = dense(h, t, p + "mlp.")
            else:
                y = moe(h, t, p + "mlp.", f,
                        choices.pop(0) if choices is not None else None)
            x = x + y
        if taps is not None:
            taps.append(x)
    return logits(x, t, cfg)
