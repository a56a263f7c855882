"""Plain, slow implementation of the Duzizen decoder, one function per mechanism, in the dtype of the weights it is given
(tests use float64 on the CPU). It keeps no cache: every call runs a whole token sequence from its start. Shares no code
with the package."""
import math

import torch


def rms(x, eps, weight=1.0):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def layer_norm(x, eps, weight, bias):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight + bias


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z**3)))


def log_sigmoid(z):
    return torch.clamp(z, max=0) - torch.log1p(torch.exp(-z.abs()))


# -----------------------------------------------------------------------------------------------
# embedding
# -----------------------------------------------------------------------------------------------
def embedding(tokens, embed, bigram, spec):
    buckets = bigram.shape[0] - 1
    rows = []
    for t, cur in enumerate(tokens):
        at = buckets if t == 0 else (tokens[t - 1] * spec["mul_prev"] + cur * spec["mul_cur"]) % buckets
        rows.append(embed[cur] + bigram[at])
    return torch.stack(rows)


# -----------------------------------------------------------------------------------------------
# rotation
# -----------------------------------------------------------------------------------------------
def frequencies(rot):
    """Angle per position of every pair."""
    n, out = rot["dims"], []
    for i in range(n // 2):
        f = rot["base"]**(-2 * i / n)
        sc = rot.get("scaling")
        if sc:
            length = 2 * math.pi / f
            if length > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif length >= sc["original"] / sc["high"]:
                s = (sc["original"] / length - sc["low"]) / (sc["high"] - sc["low"])
                f = (1 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate(x, rot, layout):
    """x [T, heads, dim]: the pairs of the first rot["dims"] dimensions turn; layout: neighbours or halves are pairs."""
    n = rot["dims"]
    y = x.clone()
    for i, f in enumerate(frequencies(rot)):
        a, b = (2 * i, 2 * i + 1) if layout == "interleaved" else (i, i + n // 2)
        ang = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * f
        c, s = torch.cos(ang).to(x.dtype), torch.sin(ang).to(x.dtype)
        y[..., a] = x[..., a] * c - x[..., b] * s
        y[..., b] = x[..., b] * c + x[..., a] * s
    return y


# -----------------------------------------------------------------------------------------------
# matrix memory with exponential gates
# -----------------------------------------------------------------------------------------------
def mlstm_scan(q, k, v, i, f):
    """q, k [T, H, d], v [T, H, e], i and f [T, H] (log gates): the read-outs [T, H, e]."""
    T, H, d = q.shape
    out = torch.zeros_like(v)
    for h in range(H):
        S, n, m = q.new_zeros(d, v.shape[2]), q.new_zeros(d), q.new_zeros(())
        for t in range(T):
            new = torch.maximum(f[t, h] + m, i[t, h])
            keep, add = torch.exp(f[t, h] + m - new), torch.exp(i[t, h] - new)
            S = keep * S + add * torch.outer(k[t, h], v[t, h])
            n = keep * n + add * k[t, h]
            m = new
            out[t, h] = (S.T @ q[t, h]) / (torch.maximum((n @ q[t, h]).abs(), torch.exp(-m)) + 1e-6)
    return out


def mlstm(h, p, m, eps):
    """p: q, k, v, i, i.b, f, f.b, norm, g, o; m: the mixer's entry of the config."""
    T = h.shape[0]
    H, d, e, cap = m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q, k, v = (h @ p["q"].T).view(T, H, d) * d**-0.5, (h @ p["k"].T).view(T, H, d), (h @ p["v"].T).view(T, H, e)
    i = cap * torch.tanh((h @ p["i"].T + p["i.b"]) / cap)
    f = log_sigmoid(cap * torch.tanh((h @ p["f"].T + p["f.b"]) / cap))
    o = rms(mlstm_scan(q, k, v, i, f), eps).reshape(T, H * e) * p["norm"]
    return (o * sigmoid(h @ p["g"].T)) @ p["o"].T


# -----------------------------------------------------------------------------------------------
# attention with short convolutions; the values are the keys
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


def sees(i, j, mask):
    if j > i:
        return False
    return not mask or not mask.get("size") or i - j < mask["size"] or j < (mask.get("keep_first") or 0)


def one_more_softmax(s):
    """exp(s_j) / (1 + sum exp(s))"""
    top = max(float(s.max()), 0.0)
    e = torch.exp(s - top)
    return e / (e.sum() + math.exp(-top))


def attention(h, p, m, eps):
    """p: q, k with their .conv and .norm, o."""
    T = h.shape[0]
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    q, k = short_conv(h @ p["q"].T, p["q.conv"]), short_conv(h @ p["k"].T, p["k.conv"])
    v = k.view(T, G, d)
    q = rotate(rms(q, eps, p["q.norm"]).view(T, H, d), m["rot"], "interleaved")
    k = rotate(rms(k, eps, p["k.norm"]).view(T, G, d), m["rot"], "interleaved")
    out = h.new_zeros(T, H, d)
    for i in range(T):
        js = [j for j in range(i + 1) if sees(i, j, m.get("mask"))]
        for a in range(H):
            b = a // (H // G)
            out[i, a] = one_more_softmax((k[js, b] @ q[i, a]) * m["scale"]) @ v[js, b]
    return out.reshape(T, H * d) @ p["o"].T


# -----------------------------------------------------------------------------------------------
# retention
# -----------------------------------------------------------------------------------------------
def retention_scan(q, k, v, decay):
    T, H, d = q.shape
    out = torch.zeros_like(v)
    for h in range(H):
        S = q.new_zeros(d, v.shape[2])
        for t in range(T):
            S = decay[h] * S + torch.outer(k[t, h], v[t, h])
            out[t, h] = S.T @ q[t, h]
    return out


def retention(h, p, m, eps):
    """p: q, k, v, g, o."""
    T = h.shape[0]
    H, d, e = m["heads"], m["dim"], m["vdim"]
    q = rotate((h @ p["q"].T).view(T, H, d), m["rot"], "half")
    k = rotate((h @ p["k"].T).view(T, H, d), m["rot"], "half") * d**-0.5
    o = rms(retention_scan(q, k, (h @ p["v"].T).view(T, H, e), m["decay"]), eps)
    return (o.reshape(T, H * e) * silu(h @ p["g"].T)) @ p["o"].T


def parallel(h, p, m, eps):
    left = attention(h, _part(p, "left."), m["left"], eps)
    right = retention(h, _part(p, "right."), m["right"], eps)
    return (rms(left, eps, p["left.out"]) + rms(right, eps, p["right.out"])) / 2


# -----------------------------------------------------------------------------------------------
# feed-forward
# -----------------------------------------------------------------------------------------------
def dense(h, p):
    return (gelu(h @ p["gate"].T) * (h @ p["up"].T)) @ p["down"].T


def expert(h, p, limit):
    g = torch.clamp(h @ p["gate"].T, max=limit)
    u = torch.clamp(h @ p["up"].T, min=-limit, max=limit)
    return (g * sigmoid(1.702 * g) * (u + 1)) @ p["down"].T


def choose(h, router, top):
    """The chosen experts of every token and their scores."""
    s = sigmoid(h @ router.T)
    best = torch.sort(s, -1, descending=True).indices[:, :top]
    return best, s.gather(1, best)


def experts(h, p, m):
    best, score = choose(h, p["router"], m["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(best[t].tolist(), score[t]):
            out[t] = out[t] + expert(w * h[t], _part(p, f"e{e}."), m["expert"]["limit"])
    return out


# -----------------------------------------------------------------------------------------------
# per-layer input of the token's own table
# -----------------------------------------------------------------------------------------------
def side(x, e, p, eps):
    """e [T, dim]: this layer's part of the tokens' rows; p: gate, proj, norm."""
    return rms((gelu(x @ p["gate"].T) * e) @ p["proj"].T, eps, p["norm"])


def _part(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens):
    """(logits [T, vocab], the residual after every layer [layers, T, width])."""
    eps, dim = cfg["norm"]["eps"], cfg["token_side"]["dim"]
    x = embedding(tokens, weights["embed"], weights["bigram"], cfg["embedding"]["bigram"])
    table = weights["side.embed"][torch.tensor(tokens)]
    trail = []

    def norm(x, name):
        return layer_norm(x, eps, weights[name], weights[name + ".b"])

    for i, e in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = norm(x, p + "norm1")
        mix = {"mlstm": mlstm, "parallel": parallel}[e["type"]]
        x = x + norm(mix(h, _part(weights, p + "mix."), e["mixer"], eps), p + "norm1b")
        if e["mlp"]:
            h, w = norm(x, p + "norm2"), _part(weights, p + "mlp.")
            y = dense(h, w) if e["mlp"].get("kind", "dense") == "dense" else experts(h, w, e["mlp"])
            x = x + norm(y, p + "norm2b")
        x = x + side(x, table[:, i * dim:(i + 1) * dim], _part(weights, p + "side."), eps)
        trail.append(x)
    return norm(x, "final.norm") @ weights["head"].T, torch.stack(trail)
