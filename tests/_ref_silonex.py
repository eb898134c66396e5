"""A plain, slow implementation of the Silonex design in float64: whole sequences, token loops,
dense masks, one function per mechanism.  It shares no code with ``lumen``; the tests compare the
framework's kernels and engine with it.

Weights are a dict {checkpoint tensor name: tensor}; the configuration is the checkpoint's
``config.json`` as a dict.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64
UNIT_EPS = 1e-6


def silu(z):
    return z / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.where(z > 0, z + torch.log1p(torch.exp(-z.abs())), torch.log1p(torch.exp(z)))


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit_vector(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + UNIT_EPS)


def short_conv(x, taps, bias=None):
    """x [T, C], taps [C, K]: y_t = sum_j taps[:, K - 1 - j] x_(t - j) (+ bias), zeros before the
    start."""
    T, K = x.shape[0], taps.shape[1]
    y = torch.zeros_like(x)
    for j in range(min(K, T)):
        y[j:] += taps[:, K - 1 - j] * x[:T - j]
    return y if bias is None else y + bias


# ---- rotary: half layout, frequencies stretched by wavelength -----------------------------------
def frequencies(rot):
    """[dims / 2] rotation per position; ``scaling``: wavelengths above original / low are
    stretched by ``factor``, those below original / high kept, a linear blend between."""
    dims, out = rot["dims"], []
    for i in range(dims // 2):
        f = float(rot["base"]) ** (-2.0 * i / dims)
        sc = rot.get("scaling")
        if sc:
            wave = 2.0 * math.pi / f
            if wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif wave >= sc["original"] / sc["high"]:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return torch.tensor(out, dtype=F64)


def rotate_half_layout(x, rot):
    """x [T, n, D]: entry i pairs with entry i + dims / 2 (i < dims / 2); the rest passes."""
    T, half = x.shape[0], rot["dims"] // 2
    a = torch.arange(T, dtype=F64).view(T, 1, 1) * frequencies(rot).view(1, 1, -1)
    c, s = torch.cos(a).to(x.dtype), torch.sin(a).to(x.dtype)
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


def window_mask(T, size):
    d = torch.arange(T).view(T, 1) - torch.arange(T).view(1, T)
    return (d >= 0) & (d < size if size else d >= 0)


# ---- the left half of a parallel mixer: window attention -----------------------------------------
def window_attention(h, w, p, m, eps):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_unit((h @ w[p + "q"].T).view(T, H, D), eps) * w[p + "q.norm"]
    k = rms_unit((h @ w[p + "k"].T).view(T, G, D), eps) * w[p + "k.norm"]
    v = rms_unit((h @ w[p + "v"].T).view(T, G, Dv), eps)
    q, k = rotate_half_layout(q, m["rot"]), rotate_half_layout(k, m["rot"])
    seen = window_mask(T, (m.get("mask") or {}).get("size"))
    out = []
    for n in range(H):
        g = n // (H // G)
        s = q[:, n] @ k[:, g].T * m["scale"]
        if m.get("softcap"):
            s = m["softcap"] * torch.tanh(s / m["softcap"])
        s = torch.where(seen, s, torch.full_like(s, -math.inf))
        out.append(torch.softmax(s, -1) @ v[:, g])
    return torch.cat(out, -1) @ w[p + "o"].T


# ---- the right half of a parallel mixer: gated delta rule -----------------------------------------
def delta_recurrence(q, k, v, beta, decay, S=None):
    """q, k [T, H, D] (one per head), v [T, H, Dv], beta, decay [T, H] -> (read-outs, state)."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if S is None else S.clone()
    out = []
    for t in range(T):
        S = decay[t].view(H, 1, 1) * S
        u = beta[t].view(H, 1) * (v[t] - (S * k[t].unsqueeze(-1)).sum(1))
        S = S + k[t].unsqueeze(-1) * u.unsqueeze(1)
        out.append((S * q[t].unsqueeze(-1)).sum(1))
    return torch.stack(out), S


def gated_delta(h, w, p, m, eps):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    conv = lambda n: silu(short_conv(h @ w[p + n].T, w[p + n + ".conv"]))  # noqa: E731
    rep = torch.arange(H) // (H // G)
    q = unit_vector(conv("q").view(T, G, D))[:, rep] * D ** -0.5
    k = unit_vector(conv("k").view(T, G, D))[:, rep]
    v = conv("v").view(T, H, Dv)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    decay = torch.exp(-torch.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    o, _ = delta_recurrence(q, k, v, beta, decay)
    o = rms_unit(o, eps) * w[p + "norm"] * silu((h @ w[p + "g"].T).view(T, H, Dv))
    return o.reshape(T, H * Dv) @ w[p + "o"].T


def parallel_mixer(h, w, p, m, eps):
    a = rms_unit(window_attention(h, w, p + "left.", m["left"], eps), eps) * w[p + "left.out"]
    b = rms_unit(gated_delta(h, w, p + "right.", m["right"], eps), eps) * w[p + "right.out"]
    return 0.5 * (a + b)


# ---- linear recurrences with a scalar decay per head -----------------------------------------------
def decayed_recurrence(q, k, v, decay, S=None):
    """q, k [T, H, D], v [T, H, Dv], decay [T, H]: S <- decay S + k v^T, o = S^T q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype) if S is None else S.clone()
    out = []
    for t in range(T):
        S = decay[t].view(H, 1, 1) * S + k[t].unsqueeze(-1) * v[t].unsqueeze(1)
        out.append((S * q[t].unsqueeze(-1)).sum(1))
    return torch.stack(out), S


def lightning(h, w, p, m, eps):
    T, H = h.shape[0], m["heads"]
    q, k, v = (silu(h @ w[p + n].T).view(T, H, -1) for n in "qkv")
    decay = torch.tensor(m["decay"], dtype=h.dtype).view(1, H).expand(T, H)
    o, _ = decayed_recurrence(q, k, v, decay)
    o = rms_unit(o.reshape(T, -1), eps) * w[p + "norm"] * torch.sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def grouped_rms(x, groups, eps):
    T, n = x.shape
    return rms_unit(x.view(T, groups, n // groups), eps).reshape(T, n)


def mamba2(h, w, p, m, eps):
    T = h.shape[0]
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    z, xbc, dt = torch.split(h @ w[p + "in"].T, [H * P, H * P + 2 * G * N, H], -1)
    xbc = silu(short_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x, B, C = torch.split(xbc, [H * P, G * N, G * N], -1)
    x = x.reshape(T, H, P)
    rep = torch.arange(H) // (H // G)
    B, C = B.reshape(T, G, N)[:, rep], C.reshape(T, G, N)[:, rep]
    dt = softplus(dt + w[p + "dt_bias"])
    decay = torch.exp(-torch.exp(w[p + "A_log"]) * dt)
    y, _ = decayed_recurrence(C, B, dt.unsqueeze(-1) * x, decay)
    y = (y + w[p + "D"].view(1, H, 1) * x).reshape(T, H * P)
    y = grouped_rms(y * silu(z), m["norm_groups"], eps) * w[p + "norm"]
    return y @ w[p + "o"].T


MIXERS = {"parallel": parallel_mixer, "lightning": lightning, "mamba2": mamba2}


def dense_ff(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


# ---- hyper-connections -----------------------------------------------------------------------------
def hyper_in(xs, w_in):
    """xs [S, T, W] -> the sublayer's input before its norm."""
    return (xs * w_in.view(-1, 1, 1)).sum(0)


def hyper_out(xs, mix, out, y):
    """New stream t: sum over the old streams s of mix[s, t] x_s, plus out[t] y."""
    return torch.stack([(xs * mix[:, t].view(-1, 1, 1)).sum(0) + out[t] * y
                        for t in range(xs.shape[0])])


def layer(xs, w, p, L, eps):
    h = layer_norm(hyper_in(xs, w[p + "hc1.in"]), w[p + "norm1"], w[p + "norm1.b"], eps)
    y = MIXERS[L["type"]](h, w, p + "mix.", L["mixer"], eps)
    xs = hyper_out(xs, w[p + "hc1.mix"], w[p + "hc1.out"], y)
    if L.get("mlp"):
        h = layer_norm(hyper_in(xs, w[p + "hc2.in"]), w[p + "norm2"], w[p + "norm2.b"], eps)
        xs = hyper_out(xs, w[p + "hc2.mix"], w[p + "hc2.out"], dense_ff(h, w, p + "mlp."))
    return xs


def layer_order(cfg):
    n = len(cfg["layers"])
    lp = cfg.get("loop")
    if not lp:
        return list(range(n))
    a, b = lp["start"], lp["stop"]
    return list(range(a)) + list(range(a, b)) * lp["times"] + list(range(b, n))


def forward(cfg, weights, tokens, layers_out=None, dtype=F64):
    """Logits [T, vocab] of one sequence from position 0, computed in ``dtype`` (float32: what
    rounding alone does to them); ``layers_out`` (a list) takes the sum of the streams after every
    layer run."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens).long()]
    xs = x.unsqueeze(0).repeat(cfg.get("streams", 1), 1, 1)
    for i in layer_order(cfg):
        xs = layer(xs, w, f"l{i}.", cfg["layers"][i], eps)
        if layers_out is not None:
            layers_out.append(xs.sum(0))
    h = layer_norm(xs.sum(0), w["final.norm"], w["final.norm.b"], eps)
    return h @ w["embed"].T * cfg.get("logit_scale", 1.0)
