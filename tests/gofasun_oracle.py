"""Plain, slow implementation of the Gofasun decoder, one function per mechanism, in the dtype of the weights it is
given (tests use float64 or float32 on the CPU). It keeps no cache: every call runs a whole token sequence from its
start, so whatever the serving engine does with pages, slots and portions is compared with a computation that has none
of them. Shares no code with the package."""
import math

import torch


def rms(x, eps, weight=None):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def input_conv(h, w):
    """h [T, C], w [C, taps]: h_t + sum_j w[:, j] h_{t - taps + 1 + j}, zeros before the start."""
    T, _ = h.shape
    taps = w.shape[1]
    out = h.clone()
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] = out[t] + w[:, j] * h[s]
    return out


def mingru(h, p, state=None):
    """h [T, C]; p: z, z.b, x, x.b, g, o. Returns (output [T, C], the state after every token [T, width])."""
    z = torch.sigmoid(h @ p["z"].T + p["z.b"])
    u = h @ p["x"].T + p["x.b"]
    cand = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    gate = h @ p["g"].T
    s = torch.zeros(z.shape[1], dtype=h.dtype) if state is None else state
    states = []
    for t in range(h.shape[0]):
        s = (1 - z[t]) * s + z[t] * cand[t]
        states.append(s)
    st = torch.stack(states) if states else h.new_zeros(0, z.shape[1])
    return (st * gate * torch.sigmoid(gate)) @ p["o"].T, st


def rotate(v, pos, dims, base):
    """Interleaved rotation of the first ``dims`` of v [..., n] at position ``pos`` (one number)."""
    out = v.clone()
    for i in range(dims // 2):
        a = pos * float(base) ** (-2.0 * i / dims)
        c, s = math.cos(a), math.sin(a)
        u, w = v[..., 2 * i], v[..., 2 * i + 1]
        out[..., 2 * i] = u * c - w * s
        out[..., 2 * i + 1] = w * c + u * s
    return out


def visible(i, j, size):
    return 0 <= i - j < size


def latent_attention(h, p, m, eps):
    """h [T, C]; p: q, dkv, dkv.norm, uk, uv, o; m: the mixer's entry of the configuration."""
    T = h.shape[0]
    H, dim, rd, vd, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    dims, base = m["rot"]["dims"], m["rot"]["base"]
    q = (h @ p["q"].T).view(T, H, dim + rd)
    down = h @ p["dkv"].T
    c = rms(down[:, :rank], eps, p["dkv.norm"])
    kr = torch.stack([rotate(down[t, rank:], t, dims, base) for t in range(T)])
    qr = torch.stack([rotate(q[t, :, dim:], t, dims, base) for t in range(T)])
    k = (c @ p["uk"].T).view(T, H, dim)
    v = (c @ p["uv"].T).view(T, H, vd)
    out = h.new_zeros(T, H, vd)
    for i in range(T):
        js = [j for j in range(T) if visible(i, j, m["mask"]["size"])]
        kj, vj, krj = k[js], v[js], kr[js]
        sc = (torch.einsum("hd,jhd->hj", q[i, :, :dim], kj) + qr[i] @ krj.T) * m["scale"]
        w = torch.exp(sc - sc.max(-1, keepdim=True).values)
        w = w / w.sum(-1, keepdim=True)
        out[i] = torch.einsum("hj,jhd->hd", w, vj)
    return out.reshape(T, H * vd) @ p["o"].T


def dense_ff(h, gate, up, down):
    return (torch.clamp(h @ gate.T, min=0) * (h @ up.T)) @ down.T


def layer_order(cfg):
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def run_layer(x, i, cfg, w):
    entry, eps, pre = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}."
    mix = {k[len(pre) + 4:]: v for k, v in w.items() if k.startswith(pre + "mix.")}
    h = input_conv(rms(x, eps) * w[pre + "norm1"], w[pre + "canon1"])
    if entry["type"] == "mingru":
        y = mingru(h, mix)[0]
    else:
        y = latent_attention(h, mix, entry["mixer"], eps)
    if entry.get("mlp"):
        f = input_conv(rms(x, eps) * w[pre + "norm2"], w[pre + "canon2"])
        y = y + dense_ff(f, w[pre + "mlp.gate"], w[pre + "mlp.up"], w[pre + "mlp.down"])
    return x + y


def forward(cfg, w, tokens):
    """tokens: list of ints. Returns (logits [T, vocab], residual stream after every layer run [runs, T, width])."""
    x = w["embed"][torch.as_tensor(tokens)]
    runs = []
    for i in layer_order(cfg):
        x = run_layer(x, i, cfg, w)
        runs.append(x)
    logits = (rms(x, cfg["norm"]["eps"]) * w["final.norm"]) @ w["head"].T
    return logits, torch.stack(runs)
