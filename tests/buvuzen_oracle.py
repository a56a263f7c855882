"""Plain, slow implementation of the Buvuzen decoder, one function per mechanism, in the dtype of the weights it is given
(tests use float64 on the CPU). It keeps no cache: every call runs a whole token sequence from its start. Shares no code
with the package."""
import torch


def rms(x, eps, weight):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def silu(z):
    return z / (1 + torch.exp(-z))


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def visible(i, j, size):
    return 0 <= i - j < size


def sink_softmax(scores, sink):
    """scores [n]; a term exp(sink) joins the sum and takes its share of the weight."""
    top = max(float(scores.max()), float(sink))
    e = torch.exp(scores - top)
    return e / (e.sum() + torch.exp(sink - top))


def attention(h, p, m, eps):
    """h [T, C]; p: q, k, v, g, o, q.norm, k.norm, sink; m: the mixer's entry of the configuration."""
    T = h.shape[0]
    H, G, d, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ p["q"].T).view(T, H, d), eps, p["q.norm"])
    k = rms((h @ p["k"].T).view(T, G, d), eps, p["k.norm"])
    v = (h @ p["v"].T).view(T, G, vd)
    gate = sigmoid(h @ p["g"].T)
    out = h.new_zeros(T, H, vd)
    for i in range(T):
        js = [j for j in range(T) if visible(i, j, m["mask"]["size"])]
        for a in range(H):
            b = a // (H // G)
            w = sink_softmax((k[js, b] @ q[i, a]) * m["scale"], p["sink"][a])
            out[i, a] = gate[i, a] * (w @ v[js, b])
    return out.reshape(T, H * vd) @ p["o"].T


def expert(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def route(z, correction, router):
    """Chosen experts of one token and their weights. z: router logits of the experts, then of the identity ones."""
    s = torch.softmax(z, -1)
    n = z.numel()
    choice = s + correction
    groups, keep = router["groups"]["count"], router["groups"]["keep"]
    size = n // groups
    best = sorted(range(groups), key=lambda g: -float(choice[g * size:(g + 1) * size].max()))[:keep]
    allowed = [e for e in range(n) if e // size in best]
    chosen = sorted(allowed, key=lambda e: -float(choice[e]))[:router["top"]]
    return chosen, [s[e] * router["scale"] for e in chosen]


def moe(h, p, mlp):
    """h [T, C]; p: router, correction, e<i>.gate / up / down, shared.gate / up / down / sg."""
    E = mlp["router"]["experts"]
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        chosen, weights = route(p["router"] @ h[t], p["correction"], mlp["router"])
        for e, w in zip(chosen, weights):
            y = h[t] if e >= E else expert(h[t], p[f"e{e}.gate"], p[f"e{e}.up"], p[f"e{e}.down"])
            out[t] = out[t] + w * y
    if mlp.get("shared"):
        sg = sigmoid(h @ p["shared.sg"].T)
        out = out + sg * expert(h, p["shared.gate"], p["shared.up"], p["shared.down"])
    return out


def _part(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens):
    """(logits [T, vocab], the residual after every layer run [runs, T, width])."""
    eps = cfg["norm"]["eps"]
    x = weights["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
    trail = []
    for i, e in enumerate(cfg["layers"]):
        while e.get("weights_of") is not None:
            i = e["weights_of"]
            e = cfg["layers"][i]
        p = f"l{i}."
        a = attention(x, _part(weights, p + "mix."), e["mixer"], eps)
        x = x + rms(a, eps, 1 + weights[p + "norm1"])
        if e["mlp"]:
            f = moe(x, _part(weights, p + "mlp."), e["mlp"])
            x = x + rms(f, eps, 1 + weights[p + "norm2"])
        trail.append(x)
    return rms(x, eps, 1 + weights["final.norm"]) @ weights["head"].T * cfg["logit_scale"], torch.stack(trail)
