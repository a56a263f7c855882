"""Prefill and decode throughput of the ragged serving engine on random weights of a real model's layer sizes: the hybrid
designs (Gofasun, Fifotar, Duzizen) next to the dense Llama layout at equal width, depth, feed-forward and head count, and
the routed designs (Buvuzen, duzizen-moe) next to the Qwen2-MoE layout at equal width, depth, heads and experts
(``bench.py --serving``). One JSON line per measurement."""
import json
import time

import torch

# name -> (width, ff, heads, kv heads of the dense model)
SIZES = {"2048": (2048, 5632, 16, 4), "4096": (4096, 14336, 32, 8)}
# name -> (experts, chosen experts, expert ff, shared expert ff) of the routed models
EXPERTS = {"2048": (64, 6, 1024, 2048), "4096": (64, 4, 2048, 4096)}
VOCAB = 32000
HEAD, ROT, WINDOW = 128, 64, 4096


def _rand(gen, dev, *shape, scale=None):
    s = shape[-1]**-0.5 if scale is None else scale
    return (torch.randn(*shape, generator=gen, device=dev, dtype=torch.float32) * s).to(torch.bfloat16)


def dense_model(size, layers, dev, max_context):
    from ..inference.v2.arch import ArchSpec
    W, ff, nq, nkv = SIZES[size]
    g = torch.Generator(device=dev).manual_seed(0)
    spec = ArchSpec("llama", VOCAB, W, layers, nq, nkv, HEAD, ff, norm_eps=1e-5, max_position_embeddings=max_context)
    one = torch.ones(W, device=dev, dtype=torch.bfloat16)
    lay = [{"ln1.w": one, "ln2.w": one, "qkv.w": _rand(g, dev, (nq + 2 * nkv) * HEAD, W),
            "o.w": _rand(g, dev, W, nq * HEAD), "up.w": _rand(g, dev, 2 * ff, W), "down.w": _rand(g, dev, W, ff)}
           for _ in range(layers)]
    return spec, {"embed": _rand(g, dev, VOCAB, W), "final.w": one, "lm_head.w": _rand(g, dev, VOCAB, W),
                  "layers": lay}


def gofasun_model(size, layers, dev, kinds=("mingru", "latent_attention")):
    from ..inference.v2.arch import convert_hf, spec_from_hf
    W, ff, H, _ = SIZES[size]
    rank = W // 8
    mixers = {"mingru": {"width": W},
              "latent_attention": {"heads": H, "dim": HEAD, "rot_dim": ROT, "kv_rank": rank, "vdim": HEAD,
                                   "scale": (HEAD + ROT)**-0.5, "rot": {"base": 10000.0, "dims": ROT},
                                   "mask": {"size": WINDOW}}}
    cfg = {"architecture": "Gofasun", "vocab": VOCAB, "width": W, "canon": {"taps": 4}, "norm": {"eps": 1e-5},
           "loop": None,
           "layers": [{"type": kinds[i % len(kinds)], "mixer": mixers[kinds[i % len(kinds)]],
                       "mlp": {"kind": "dense", "ff": ff}} for i in range(layers)]}
    g = torch.Generator(device=dev).manual_seed(0)
    w = {"embed": _rand(g, dev, VOCAB, W), "head": _rand(g, dev, VOCAB, W), "final.norm": torch.ones((), device=dev)}
    for i, e in enumerate(cfg["layers"]):
        p = f"l{i}."
        for k in ("1", "2"):
            w[p + "norm" + k] = torch.ones((), device=dev)
            w[p + "canon" + k] = _rand(g, dev, W, cfg["canon"]["taps"], scale=0.1)
        shapes = {"mlp.gate": (ff, W), "mlp.up": (ff, W), "mlp.down": (W, ff)}
        if e["type"] == "mingru":
            shapes.update({"mix.z": (W, W), "mix.x": (W, W), "mix.g": (W, W), "mix.o": (W, W)})
            w[p + "mix.z.b"] = _rand(g, dev, W, scale=1.0)
            w[p + "mix.x.b"] = _rand(g, dev, W, scale=1.0)
        else:
            shapes.update({"mix.q": (H * (HEAD + ROT), W), "mix.dkv": (rank + ROT, W), "mix.uk": (H * HEAD, rank),
                           "mix.uv": (H * HEAD, rank), "mix.o": (W, H * HEAD)})
            w[p + "mix.dkv.norm"] = torch.ones(rank, device=dev)
        for k, s in shapes.items():
            w[p + k] = _rand(g, dev, *s)
    spec = spec_from_hf(cfg)
    return spec, convert_hf(w, spec)


def moe_model(size, layers, dev, max_context):
    from ..inference.v2.arch import ArchSpec
    W, _, nq, nkv = SIZES[size]
    E, top, ff, sh = EXPERTS[size]
    g = torch.Generator(device=dev).manual_seed(0)
    spec = ArchSpec("qwen2_moe", VOCAB, W, layers, nq, nkv, HEAD, ff, norm_eps=1e-5, sliding_window=WINDOW,
                    max_position_embeddings=max_context,
                    moe=dict(num_experts=E, top_k=top, normalize=False, shared=True, shared_intermediate_size=sh))
    one = torch.ones(W, device=dev, dtype=torch.bfloat16)
    lay = [{"ln1.w": one, "ln2.w": one, "qkv.w": _rand(g, dev, (nq + 2 * nkv) * HEAD, W),
            "o.w": _rand(g, dev, W, nq * HEAD), "router.w": _rand(g, dev, E, W), "w13": _rand(g, dev, E, 2 * ff, W),
            "w2": _rand(g, dev, E, W, ff), "shared.w13": _rand(g, dev, 2 * sh, W), "shared.w2": _rand(g, dev, W, sh),
            "shared_gate.w": _rand(g, dev, 1, W)} for _ in range(layers)]
    return spec, {"embed": _rand(g, dev, VOCAB, W), "final.w": one, "lm_head.w": _rand(g, dev, VOCAB, W),
                  "layers": lay}


def buvuzen_model(size, layers, dev):
    from ..inference.v2.arch import convert_hf, spec_from_hf
    W, _, nq, nkv = SIZES[size]
    E, top, ff, sh = EXPERTS[size]
    layer = {"type": "attention",
             "mixer": {"heads": nq, "kv_heads": nkv, "dim": HEAD, "vdim": HEAD, "scale": HEAD**-0.5,
                       "mask": {"size": WINDOW}},
             "mlp": {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": sh},
                     "router": {"experts": E, "identity": 0, "top": top, "groups": {"count": 8, "keep": 4},
                                "scale": 2.0}}}
    cfg = {"architecture": "Buvuzen", "vocab": VOCAB, "width": W, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0},
           "logit_scale": 1.0, "layers": [layer] * layers}
    g = torch.Generator(device=dev).manual_seed(0)
    w = {"embed": _rand(g, dev, VOCAB, W), "head": _rand(g, dev, VOCAB, W), "final.norm": torch.zeros(W, device=dev)}
    for i in range(layers):
        p = f"l{i}."
        for k, n in (("norm1", W), ("norm2", W), ("mix.sink", nq), ("mlp.correction", E)):
            w[p + k] = torch.zeros(n, device=dev)
        for k in ("mix.q.norm", "mix.k.norm"):
            w[p + k] = torch.ones(HEAD, device=dev)
        shapes = {"mix.q": (nq * HEAD, W), "mix.k": (nkv * HEAD, W), "mix.v": (nkv * HEAD, W), "mix.g": (nq, W),
                  "mix.o": (W, nq * HEAD), "mlp.router": (E, W), "mlp.shared.gate": (sh, W), "mlp.shared.up": (sh, W),
                  "mlp.shared.down": (W, sh), "mlp.shared.sg": (1, W)}
        for e in range(E):
            shapes.update({f"mlp.e{e}.gate": (ff, W), f"mlp.e{e}.up": (ff, W), f"mlp.e{e}.down": (W, ff)})
        for k, s in shapes.items():
            w[p + k] = _rand(g, dev, *s)
    spec = spec_from_hf(cfg)
    return spec, convert_hf(w, spec)


FIFOTAR = ("attention", "delta", "latent_attention", "delta")


def fifotar_model(size, layers, dev, kinds=FIFOTAR):
    from ..inference.v2.arch import convert_hf, spec_from_hf
    W, ff, H, G = SIZES[size]
    rank, qrank, taps = W // 8, W // 4, 4
    mixers = {"delta": {"heads": H, "kv_heads": H // 2, "dim": HEAD, "vdim": HEAD, "conv": taps},
              "latent_attention": {"heads": H, "dim": HEAD, "rot_dim": ROT, "kv_rank": rank, "q_rank": qrank,
                                   "vdim": HEAD, "scale": (HEAD + ROT)**-0.5,
                                   "rot": {"base": 500000.0, "dims": ROT, "scaling": {
                                       "factor": 8.0, "fast": 32.0, "slow": 1.0, "original": 4096}}},
              # as many keys as the other models see
              "attention": {"heads": H, "kv_heads": G, "dim": HEAD, "vdim": HEAD, "scale": HEAD**-0.5, "softcap": 50.0,
                            "v_mix": True, "mask": {"size": 2 * WINDOW}}}
    cfg = {"architecture": "Fifotar", "vocab": VOCAB, "width": W, "norm": {"eps": 1e-5}, "embedding": {"scale": W**0.5},
           "residual_mult": 0.5, "logit_softcap": 30.0,
           "layers": [{"type": kinds[i % len(kinds)], "mixer": mixers[kinds[i % len(kinds)]],
                       "mlp": {"kind": "dense", "ff": ff, "limit": 7.0}} for i in range(layers)]}
    g = torch.Generator(device=dev).manual_seed(0)
    w = {"embed": _rand(g, dev, VOCAB, W), "final.norm": torch.ones(W, device=dev)}
    for i, e in enumerate(cfg["layers"]):
        p, m = f"l{i}.", e["mixer"]
        for k in ("norm1", "norm1b", "norm2", "norm2b"):
            w[p + k] = torch.ones(W, device=dev)
        shapes = {"mlp.gate": (ff, W), "mlp.up": (ff, W), "mlp.down": (W, ff), "mix.o": (W, H * HEAD)}
        if e["type"] == "delta":
            D = H // 2 * HEAD
            shapes.update({"mix.q": (D, W), "mix.k": (D, W), "mix.v": (H * HEAD, W), "mix.g": (H * HEAD, W),
                           "mix.b": (H, W), "mix.a": (H, W)})
            for k, n in (("q", D), ("k", D), ("v", H * HEAD)):
                w[f"{p}mix.{k}.conv"] = _rand(g, dev, n, taps, scale=0.5)
            w[p + "mix.A_log"], w[p + "mix.dt_bias"] = _rand(g, dev, H, scale=1.0), _rand(g, dev, H, scale=1.0)
            w[p + "mix.norm"] = torch.ones(HEAD, device=dev)
        elif e["type"] == "latent_attention":
            shapes.update({"mix.dq": (qrank, W), "mix.uq": (H * (HEAD + ROT), qrank), "mix.dkv": (rank + ROT, W),
                           "mix.uk": (H * HEAD, rank), "mix.uv": (H * HEAD, rank), "mix.g": (H, W)})
            w[p + "mix.dq.norm"], w[p + "mix.dkv.norm"] = torch.ones(qrank, device=dev), torch.ones(rank, device=dev)
        else:
            shapes.update({"mix.q": (H * HEAD, W), "mix.k": (G * HEAD, W), "mix.v": (G * HEAD, W),
                           "mix.g": (H * HEAD, W)})
            w[p + "mix.vmix"] = torch.tensor(0.5, device=dev)
        for k, s in shapes.items():
            w[p + k] = _rand(g, dev, *s)
    spec = spec_from_hf(cfg)
    return spec, convert_hf(w, spec)


DUZIZEN = ("mlstm", "parallel")
KEPT, SIDE, BUCKETS = 64, 256, 32768


def duzizen_model(size, layers, dev, kinds=DUZIZEN, routed=False):
    """A parallel layer has half of the heads in each of its mixers."""
    from ..inference.v2.arch import convert_hf, spec_from_hf
    W, ff, H, G = SIZES[size]
    E, top, eff, _ = EXPERTS[size]
    taps, h, g2 = 4, H // 2, G // 2
    mixers = {"mlstm": {"heads": H, "dim": HEAD, "vdim": HEAD, "gate_cap": 15.0},
              "parallel": {"left": {"heads": h, "kv_heads": g2, "dim": HEAD, "vdim": HEAD, "conv": taps, "scale": HEAD**-0.5,
                                    "mask": {"size": WINDOW, "keep_first": KEPT},
                                    "rot": {"base": 500000.0, "dims": ROT, "scaling": {
                                        "factor": 8.0, "low": 1.0, "high": 4.0, "original": 4096}}},
                           "right": {"heads": h, "dim": HEAD, "vdim": HEAD, "decay": [1 - 0.5**(5 + 0.25 * i) for i in range(h)],
                                     "rot": {"base": 10000.0, "dims": HEAD}}}}
    mlp = {"kind": "moe", "router": {"experts": E, "top": top}, "expert": {"ff": eff, "limit": 7.0}} if routed else \
        {"kind": "dense", "ff": ff}
    cfg = {"architecture": "Duzizen", "vocab": VOCAB, "width": W, "norm": {"eps": 1e-5}, "token_side": {"dim": SIDE},
           "embedding": {"bigram": {"buckets": BUCKETS, "mul_prev": 7919, "mul_cur": 31}},
           "layers": [{"type": kinds[i % len(kinds)], "mixer": mixers[kinds[i % len(kinds)]], "mlp": mlp}
                      for i in range(layers)]}
    g = torch.Generator(device=dev).manual_seed(0)
    one, zero = torch.ones(W, device=dev), torch.zeros(W, device=dev)
    w = {"embed": _rand(g, dev, VOCAB, W), "head": _rand(g, dev, VOCAB, W), "bigram": _rand(g, dev, BUCKETS + 1, W),
         "side.embed": _rand(g, dev, VOCAB, SIDE * layers, scale=1.0), "final.norm": one, "final.norm.b": zero}
    for i, e in enumerate(cfg["layers"]):
        p = f"l{i}."
        for k in ("norm1", "norm1b", "norm2", "norm2b"):
            w[p + k], w[p + k + ".b"] = one, zero
        w[p + "side.norm"] = one
        shapes = {"side.gate": (SIDE, W), "side.proj": (W, SIDE)}
        if routed:
            shapes["mlp.router"] = (E, W)
            for x in range(E):
                shapes.update({f"mlp.e{x}.gate": (eff, W), f"mlp.e{x}.up": (eff, W), f"mlp.e{x}.down": (W, eff)})
        else:
            shapes.update({"mlp.gate": (ff, W), "mlp.up": (ff, W), "mlp.down": (W, ff)})
        if e["type"] == "mlstm":
            shapes.update({f"mix.{k}": (H * HEAD, W) for k in "qkvg"})
            shapes.update({"mix.o": (W, H * HEAD), "mix.i": (H, W), "mix.f": (H, W)})
            w[p + "mix.norm"] = torch.ones(H * HEAD, device=dev)
            w[p + "mix.i.b"], w[p + "mix.f.b"] = torch.zeros(H, device=dev), torch.full((H, ), 4.0, device=dev)
        else:
            for k, n in (("q", h * HEAD), ("k", g2 * HEAD)):
                shapes[f"mix.left.{k}"] = (n, W)
                w[f"{p}mix.left.{k}.conv"] = _rand(g, dev, n, taps, scale=0.5)
                w[f"{p}mix.left.{k}.norm"] = torch.ones(n, device=dev)
            shapes.update({f"mix.right.{k}": (h * HEAD, W) for k in "qkvg"})
            shapes.update({"mix.left.o": (W, h * HEAD), "mix.right.o": (W, h * HEAD)})
            w[p + "mix.left.out"], w[p + "mix.right.out"] = one, one
        for k, s in shapes.items():
            w[p + k] = _rand(g, dev, *s)
    spec = spec_from_hf(cfg)
    return spec, convert_hf(w, spec)


def _engine(kind, size, layers, dev, batch, max_context, max_batch_tokens):
    from ..inference.v2.engine import InferenceEngineV2, RaggedInferenceEngineConfig
    if kind == "llama":
        spec, w = dense_model(size, layers, dev, max_context)
    elif kind == "qwen2-moe":
        spec, w = moe_model(size, layers, dev, max_context)
    elif kind == "buvuzen":
        spec, w = buvuzen_model(size, layers, dev)
    elif kind.startswith("fifotar"):
        kinds = {"fifotar": FIFOTAR, "fifotar-delta": ("delta", ), "fifotar-latent": ("latent_attention", ),
                 "fifotar-attention": ("attention", )}[kind]
        spec, w = fifotar_model(size, layers, dev, kinds)
    elif kind.startswith("duzizen"):
        kinds = {"duzizen-mlstm": ("mlstm", ), "duzizen-parallel": ("parallel", )}.get(kind, DUZIZEN)
        spec, w = duzizen_model(size, layers, dev, kinds, routed=kind == "duzizen-moe")
    else:
        kinds = {"gofasun": ("mingru", "latent_attention"), "gofasun-mingru": ("mingru", ),
                 "gofasun-latent": ("latent_attention", )}[kind]
        spec, w = gofasun_model(size, layers, dev, kinds)
    conf = RaggedInferenceEngineConfig.from_dict(dict(
        dtype="bf16", state_manager=dict(max_context=max_context, max_ragged_batch_size=max_batch_tokens,
                                         max_tracked_sequences=max(4, batch), kv_block_size=64)))
    return InferenceEngineV2(spec, w, conf, device=dev, num_kv_blocks=batch * (-(-max_context // 64)))


def _time(fn, steps, warmup):
    for _ in range(warmup):
        fn()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(steps):
        fn()
    torch.cuda.synchronize()
    return (time.perf_counter() - t0) / steps


def measure(kind, size, layers, dev, prompt, batches, steps, warmup):
    g = torch.Generator().manual_seed(1)
    top = max(batches)
    ctx = prompt + 64 * (1 + (2 * (steps + warmup) + 8) // 64)
    eng = _engine(kind, size, layers, dev, top, ctx, prompt)
    ids = torch.randint(0, VOCAB, (prompt, ), generator=g)
    base = {"model": kind, "width": int(size), "layers": layers}

    def prefill():
        eng.put(["p"], [ids], capture_latents=False)
        eng.flush("p")

    dt = _time(prefill, max(2, steps // 4), 2)
    yield dict(base, phase="prefill", tokens=prompt, ms=round(dt * 1e3, 3), tok_per_s=round(prompt / dt, 1))
    for B in batches:
        uids = list(range(B))
        for u in uids:
            eng.put([u], [ids], capture_latents=False)
        tok = [torch.tensor([5 + u]) for u in uids]
        dt = _time(lambda: eng.put(uids, tok, capture_latents=False), steps, warmup)
        for u in uids:
            eng.flush(u)
        yield dict(base, phase="decode", batch=B, context=prompt, ms=round(dt * 1e3, 3), tok_per_s=round(B / dt, 1))


def run(models=("llama", "gofasun"), sizes=("2048", "4096"), layers=8, prompt=4096, batches=(1, 4, 16), steps=32,
        warmup=4):
    dev = torch.device("cuda", 0)
    for size in sizes:
        for kind in models:
            for rec in measure(kind, size, layers, dev, prompt, batches, steps, warmup):
                print(json.dumps(rec), flush=True)
            torch.cuda.empty_cache()
