"""A plain, slow implementation of the Tazulix design in float64: whole sequences, token loops,
dense masks, one function per mechanism.  It shares no code with ``lumen``; the tests compare the
framework's kernels and engine with it.

Weights are a dict {checkpoint tensor name: tensor}; the configuration is the checkpoint's
``config.json`` as a dict.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64
GATE_SLOPE = 1.702


def silu(z):
    return z / (1.0 + torch.exp(-z))


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


# ---- rotary: half layout, YaRN ---------------------------------------------------------------------
def frequencies(rot):
    """([dims / 2] rotation per position, factor on cosine and sine)."""
    dims, base = rot["dims"], float(rot["base"])
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(plain, dtype=F64), 1.0

    def dim_of(turns):
        """The (fractional) dimension whose wavelength fits ``turns`` times into the original
        context."""
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(dim_of(sc["fast"])), 0)
    hi = min(math.ceil(dim_of(sc["slow"])), dims - 1)
    out = []
    for i, f in enumerate(plain):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / sc["factor"] * ramp + f * (1.0 - ramp))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, pos, rot):
    """x [T, n, D] at positions pos [T]: entry i pairs with entry i + dims / 2; the rest passes."""
    half = rot["dims"] // 2
    f, amp = frequencies(rot)
    a = torch.as_tensor(pos).to(F64).view(-1, 1, 1) * f.view(1, 1, -1)
    c, s = (torch.cos(a) * amp).to(x.dtype), (torch.sin(a) * amp).to(x.dtype)
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


def causal_attention(q, k, v, scale):
    """q [T, H, D], k [T, G, D], v [T, G, Dv] -> [T, H, Dv]."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    seen = torch.ones(T, T).tril().bool()
    out = []
    for n in range(H):
        g = n // (H // G)
        s = q[:, n] @ k[:, g].T * scale
        s = torch.where(seen, s, torch.full_like(s, -math.inf))
        out.append(torch.softmax(s, -1) @ v[:, g])
    return torch.stack(out, 1)


def attention(h, w, p, m, eps):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    proj = lambda n: h @ w[p + n].T + w[p + n + ".b"]  # noqa: E731
    q = (rms_unit(proj("q"), eps) * w[p + "q.norm"]).view(T, H, D)
    k = (rms_unit(proj("k"), eps) * w[p + "k.norm"]).view(T, G, D)
    pos = torch.arange(T)
    o = causal_attention(rotate(q, pos, m["rot"]), rotate(k, pos, m["rot"]),
                         proj("v").view(T, G, Dv), m["scale"])
    return o.reshape(T, H * Dv) @ w[p + "o"].T


# ---- linear recurrence with a constant decay per head -----------------------------------------------
def decayed_recurrence(q, k, v, decay, S=None):
    """q, k [T, H, D], v [T, H, Dv], decay [H]: S <- decay S + k v^T, o = S^T q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if S is None else S.clone()
    out = []
    for t in range(T):
        S = decay.view(H, 1, 1) * S + k[t].unsqueeze(-1) * v[t].unsqueeze(1)
        out.append((S * q[t].unsqueeze(-1)).sum(1))
    return torch.stack(out), S


def lightning(h, w, p, m, eps):
    T, H = h.shape[0], m["heads"]
    q, k, v = (silu(h @ w[p + n].T).view(T, H, -1) for n in "qkv")
    o, _ = decayed_recurrence(q, k, v, torch.tensor(m["decay"], dtype=h.dtype))
    o = rms_unit(o.reshape(T, -1), eps) * w[p + "norm"] * torch.sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


# ---- feed-forwards -----------------------------------------------------------------------------------
def dense_ff(h, w, p, f):
    return torch.clamp(h @ w[p + "up"].T, min=0.0) ** 2 @ w[p + "down"].T


def expert(h, w, p, limit):
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(GATE_SLOPE * g) * (u + 1.0)) @ w[p + "down"].T


def route(z, top):
    """Router logits [T, E] -> weights [T, E]: the ``top`` largest sigmoids as they are, 0 elsewhere."""
    s = torch.sigmoid(z)
    out = torch.zeros_like(s)
    for t in range(s.shape[0]):
        for e in sorted(range(s.shape[1]), key=lambda e: (-float(s[t, e]), e))[:top]:
            out[t, e] = s[t, e]
    return out


def moe_ff(h, w, p, f):
    wt = route(h @ w[p + "router"].T, f["router"]["top"])
    y = torch.zeros_like(h)
    for e in range(f["router"]["experts"]):
        rows = torch.nonzero(wt[:, e] > 0).flatten()
        if rows.numel():
            y[rows] += expert(wt[rows, e, None] * h[rows], w, p + f"e{e}.", f["expert"]["limit"])
    if f.get("shared"):
        y = y + expert(h, w, p + "shared.", f["shared"]["limit"])
    return y


MIXERS = {"attention": attention, "lightning": lightning}
FEED_FORWARDS = {"dense": dense_ff, "moe": moe_ff}


def layer(x, w, p, L, eps):
    h = rms_unit(x, eps) * w[p + "norm1"]
    x = x + MIXERS[L["type"]](h, w, p + "mix.", L["mixer"], eps)
    f = L.get("mlp")
    if f:
        h = rms_unit(x, eps) * w[p + "norm2"]
        x = x + FEED_FORWARDS[f["kind"]](h, w, p + "mlp.", f)
    return x


def loop_input(x, x0, w):
    return torch.cat([x, x0], -1) @ w["loop.in"].T


def layer_order(cfg):
    """[(layer, does a pass begin with it)] in the order they run."""
    n = len(cfg["layers"])
    lp = cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    a, b = lp["start"], lp["stop"]
    return ([(i, False) for i in range(a)] + [(i, i == a) for i in range(a, b)] * lp["times"]
            + [(i, False) for i in range(b, n)])


def forward(cfg, weights, tokens, layers_out=None, dtype=F64):
    """Logits [T, vocab] of one sequence from position 0, computed in ``dtype`` (float32: what
    rounding alone does to them); ``layers_out`` (a list) takes the stream after every layer run."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x0 = w["embed"][torch.as_tensor(tokens).long()] * cfg["embedding"]["scale"]
    x = x0
    for i, enter in layer_order(cfg):
        if enter:
            x = loop_input(x, x0, w)
        x = layer(x, w, f"l{i}.", cfg["layers"][i], eps)
        if layers_out is not None:
            layers_out.append(x)
    return (rms_unit(x, eps) * w["final.norm"]) @ w["head"].T
