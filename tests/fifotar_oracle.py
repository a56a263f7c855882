"""Plain, slow implementation of the Fifotar decoder, one function per mechanism, in the dtype of the weights it is given
(tests use float64 on the CPU). It keeps no cache: every call runs a whole token sequence from its start. Shares no code
with the package."""
import math

import torch


def rms(x, eps, weight=1.0):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def softcap(z, cap):
    return cap * torch.tanh(z / cap) if cap else z


# -----------------------------------------------------------------------------------------------
# gated delta rule
# -----------------------------------------------------------------------------------------------
def short_conv(x, w):
    """x [T, C]; w [C, taps], the newest input in the last column."""
    T, taps = x.shape[0], w.shape[1]
    y = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                y[t] = y[t] + w[:, j] * x[s]
    return y


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_scan(q, k, v, decay, beta):
    """q, k [T, H, d], v [T, H, e], decay and beta [T, H]: the read-outs [T, H, e]."""
    T, H, d = q.shape
    out = torch.zeros_like(v)
    for h in range(H):
        S = q.new_zeros(d, v.shape[2])
        for t in range(T):
            S = decay[t, h] * S
            u = beta[t, h] * (v[t, h] - S.T @ k[t, h])
            S = S + torch.outer(k[t, h], u)
            out[t, h] = S.T @ q[t, h]
    return out


def delta(h, p, m, eps):
    """h [T, C]; p: q, k, v with their .conv, b, a, A_log, dt_bias, norm, g, o; m: the mixer's entry of the config."""
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(short_conv(h @ p["q"].T, p["q.conv"])).view(T, G, d)
    k = silu(short_conv(h @ p["k"].T, p["k.conv"])).view(T, G, d)
    v = silu(short_conv(h @ p["v"].T, p["v.conv"])).view(T, H, e)
    group = torch.arange(H) // (H // G)
    q, k = unit(q)[:, group] * d**-0.5, unit(k)[:, group]
    beta = sigmoid(h @ p["b"].T)
    decay = torch.exp(-torch.exp(p["A_log"]) * softplus(h @ p["a"].T + p["dt_bias"]))
    o = rms(delta_scan(q, k, v, decay, beta), eps, p["norm"])
    return (o * silu(h @ p["g"].T).view(T, H, e)).reshape(T, H * e) @ p["o"].T


# -----------------------------------------------------------------------------------------------
# latent attention
# -----------------------------------------------------------------------------------------------
def frequencies(rot):
    """(angle per position of every pair, factor of cos and sin)."""
    n, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    out = []
    for i in range(n // 2):
        f = base**(-2 * i / n)
        if sc:
            def turns_to_dim(t):
                return n * math.log(sc["original"] / (2 * math.pi * t)) / (2 * math.log(base))
            lo = max(math.floor(turns_to_dim(sc["fast"])), 0)
            hi = min(math.ceil(turns_to_dim(sc["slow"])), n - 1)
            ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            f = f / sc["factor"] * ramp + f * (1 - ramp)
        out.append(f)
    return out, (0.1 * math.log(sc["factor"]) + 1 if sc else 1.0)


def rotate(x, rot):
    """x [T, ..., rot dims]: pair (i, i + half) of the first rot["dims"] turns by its angle at every position."""
    n = rot["dims"]
    freq, mul = frequencies(rot)
    y = x.clone()
    for t in range(x.shape[0]):
        for i in range(n // 2):
            a = t * freq[i]
            c, s = mul * math.cos(a), mul * math.sin(a)
            u, w = x[t, ..., i], x[t, ..., i + n // 2]
            y[t, ..., i] = u * c - w * s
            y[t, ..., i + n // 2] = w * c + u * s
    return y


def latent_attention(h, p, m, eps):
    """p: dq, dq.norm, uq, dkv, dkv.norm, uk, uv, g, o."""
    T = h.shape[0]
    H, d, r, e, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (rms(h @ p["dq"].T, eps, p["dq.norm"]) @ p["uq"].T).view(T, H, d + r)
    ckv = h @ p["dkv"].T
    c = rms(ckv[:, :rank], eps, p["dkv.norm"])
    kr = rotate(ckv[:, rank:], m["rot"])
    qr = rotate(q[..., d:], m["rot"])
    k, v = (c @ p["uk"].T).view(T, H, d), (c @ p["uv"].T).view(T, H, e)
    gate = sigmoid(h @ p["g"].T)
    out = h.new_zeros(T, H, e)
    for i in range(T):
        for a in range(H):
            s = (k[:i + 1, a] @ q[i, a, :d] + kr[:i + 1] @ qr[i, a]) * m["scale"]
            out[i, a] = gate[i, a] * (torch.softmax(s, 0) @ v[:i + 1, a])
    return out.reshape(T, H * e) @ p["o"].T


# -----------------------------------------------------------------------------------------------
# chunked attention
# -----------------------------------------------------------------------------------------------
def first_visible(i, size):
    """The first position that position i sees."""
    return i - i % size if size else 0


def one_more_softmax(s):
    """exp(s_j) / (1 + sum exp(s))"""
    top = max(float(s.max()), 0.0)
    e = torch.exp(s - top)
    return e / (e.sum() + math.exp(-top))


def attention(h, p, m, first=None):
    """p: q, k, v, g, o and vmix; first: the values [T, G, vdim] to mix in, or None. Returns (output, own values)."""
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k = (h @ p["q"].T).view(T, H, d), (h @ p["k"].T).view(T, G, d)
    own = (h @ p["v"].T).view(T, G, e)
    v = own if first is None else (1 - p["vmix"]) * own + p["vmix"] * first
    out = h.new_zeros(T, H, e)
    for i in range(T):
        j = first_visible(i, (m.get("mask") or {}).get("size"))
        for a in range(H):
            b = a // (H // G)
            s = softcap((k[j:i + 1, b] @ q[i, a]) * m["scale"], m.get("softcap"))
            out[i, a] = one_more_softmax(s) @ v[j:i + 1, b]
    return (out.reshape(T, H * e) * sigmoid(h @ p["g"].T)) @ p["o"].T, own


# -----------------------------------------------------------------------------------------------
def feed_forward(h, p, limit):
    g = torch.clamp(h @ p["gate"].T, max=limit)
    u = torch.clamp(h @ p["up"].T, min=-limit, max=limit)
    return (g * sigmoid(1.702 * g) * (u + 1)) @ p["down"].T


def _part(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens):
    """(logits [T, vocab], the residual after every layer [layers, T, width])."""
    eps, mul = cfg["norm"]["eps"], cfg["residual_mult"]
    x = weights["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
    trail, first = [], None
    for i, e in enumerate(cfg["layers"]):
        w, m = _part(weights, f"l{i}."), e["mixer"]
        p, h = _part(w, "mix."), rms(x, eps, w["norm1"])
        if e["type"] == "delta":
            y = delta(h, p, m, eps)
        elif e["type"] == "latent_attention":
            y = latent_attention(h, p, m, eps)
        else:
            mixes = bool(m.get("v_mix"))
            y, own = attention(h, p, m, first if mixes else None)
            if mixes and first is None:
                first = own
        x = x + mul * rms(y, eps, w["norm1b"])
        if e["mlp"]:
            y = feed_forward(rms(x, eps, w["norm2"]), _part(w, "mlp."), e["mlp"]["limit"])
            x = x + mul * rms(y, eps, w["norm2b"])
        trail.append(x)
    logits = rms(x, eps, weights["final.norm"]) @ weights["embed"].T
    return softcap(logits, cfg["logit_softcap"]), torch.stack(trail)
