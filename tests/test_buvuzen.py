"""Buvuzen on the ragged serving engine against the plain implementation in buvuzen_oracle.py: every mechanism alone, then
the engine with whole prompts, portions, single tokens, mixed batches, reused pages and slots, decode graphs, eviction,
tensor parallelism, serialization, generation and trace replay. CPU runs use the ops' torch implementations, ``gpu`` runs
the HIP kernels in 32-bit and in bfloat16."""
import json
import math
import os
import re

import pytest
import torch

from hcache_deepspeed_amd.inference.v2 import build_engine_from_ds_checkpoint, build_hf_engine
from hcache_deepspeed_amd.inference.v2.arch import convert_hf, run_order, spec_from_hf
from hcache_deepspeed_amd.inference.v2.engine import (InferenceEngineV2, RaggedInferenceEngineConfig, SchedulingError,
                                                      transformer_class)
from hcache_deepspeed_amd.inference.v2.modules import DSExpertLayerConfig, instantiate_expert_layer
from hcache_deepspeed_amd.ops import experts as experts_op
from hcache_deepspeed_amd.ops.experts import RouterShape, route, routed_experts
from hcache_deepspeed_amd.ops.output_norm import embed_rows, norm_rows, residual_norm, sum_experts
from hcache_deepspeed_amd.ops.paged import HeadShape, head_attention, head_blocks_ok, make_head_plan

from . import buvuzen_oracle as oracle
from .serving_utils import GPU, Pages, close, feed, portions, rnd, run, tokens  # noqa: F401

# -----------------------------------------------------------------------------------------------
# attention
# -----------------------------------------------------------------------------------------------
# (heads, kv heads, dim, vdim, window): sizes of the plain kernel, of the exact and of the zero-padded tiles
SHAPES = {"odd": (3, 1, 5, 7, 11), "odd-gqa": (6, 2, 12, 20, 19), "exact-64": (4, 2, 64, 64, 33),
          "exact-80": (2, 2, 80, 80, 0), "exact-128": (8, 1, 128, 128, 40), "padded-40": (5, 5, 40, 40, 21),
          "uneven": (6, 3, 24, 56, 70), "uneven-wide": (4, 1, 136, 72, 50), "uneven-value": (2, 1, 16, 200, 18),
          "12-per-key": (12, 1, 32, 32, 64), "window-1": (3, 3, 16, 16, 1), "256": (2, 1, 256, 256, 30),
          "plain-wide": (2, 2, 264, 24, 25)}


def _shape(name, gated=True):
    H, G, d, vd, win = SHAPES[name]
    sh = HeadShape(heads=H, kv_heads=G, dim=d, vdim=vd, window=win, scale=1.7 / math.sqrt(d), eps=1e-4, gated=gated)
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": vd, "scale": sh.scale, "mask": {"size": win or 10**9}}
    return sh, m


def _norms(sh, seed=4):
    return {"q.norm": 1 + 0.3 * rnd(sh.dim, seed=seed), "k.norm": 1 + 0.3 * rnd(sh.dim, seed=seed + 1),
            "sink": rnd(sh.heads, seed=seed + 2)}


def _run_heads(sh, qkvs, w, sizes, dev, dtype, decode_max=None, block_size=16):
    """The op over portions of several sequences; returns every sequence's outputs."""
    lengths = [q.shape[0] for q in qkvs]
    blocks = len(qkvs) * (-(-max(lengths) // block_size) + 1)
    pages = Pages(len(qkvs), blocks, block_size, sh.row, list(range(len(qkvs)))[::-1], dev, dtype)
    f = {k: None if v is None else v.float().to(dev) for k, v in w.items()}
    outs = [[] for _ in qkvs]
    ld = -(-sh.width // 8) * 8
    for step in portions(lengths, sizes):
        b = pages.batch(step)
        x = torch.cat([qkvs[s][p:p + n] for s, n, p in step])
        qkv = torch.full((x.shape[0], ld), float("nan"), dtype=dtype, device=dev)
        qkv[:, :sh.width] = x.to(dtype).to(dev)
        out = torch.zeros(x.shape[0], sh.heads * sh.vdim + 8, dtype=dtype, device=dev)
        blocks_on = dev.type == "cuda" and b.max_new > 1 and head_blocks_ok(sh, dtype)
        plan = make_head_plan(b.seq_meta_host, b.current_tokens, sh.heads, sh.kv_heads, blocks_on, dev, decode_max)
        head_attention(qkv, sh, f["q.norm"], f["k.norm"], f["sink"], pages.cache, b, plan,
                       out[:, :sh.heads * sh.vdim])
        assert (out[:, sh.heads * sh.vdim:] == 0).all()
        for i, (s, n, _) in enumerate(step):
            q0 = b.seq_meta_host[i][0]
            outs[s].append(out[q0:q0 + n, :sh.heads * sh.vdim].double().cpu())
    return [torch.cat(o) for o in outs]


def _oracle_heads(sh, m, qkv, w):
    """The oracle on the projected rows: its projections pick them out."""
    eye = torch.eye(sh.width, dtype=torch.float64)
    q, k, v, g = eye.split([sh.heads * sh.dim, sh.kv_heads * sh.dim, sh.kv_heads * sh.vdim,
                            sh.width - sh.qkv_width])
    return oracle.attention(qkv, {"q": q, "k": k, "v": v, "g": g, "o": torch.eye(sh.heads * sh.vdim).double(), **w}, m,
                            sh.eps)


@pytest.mark.parametrize("name", list(SHAPES))
@pytest.mark.parametrize("sizes", [[1000], [1], [2], [37, 1, 5, 2, 64, 90]])
def test_attention(run, name, sizes):
    dev, dtype = run
    sh, m = _shape(name)
    w = _norms(sh)
    qkvs = [rnd(n, sh.width, seed=40 + n).to(dtype).double() for n in (75, 2, 41)]
    got = _run_heads(sh, qkvs, w, sizes, dev, dtype)
    for g, x in zip(got, qkvs):
        close(g, _oracle_heads(sh, m, x, w), dtype, bf16=2e-2)


@pytest.mark.parametrize("name", ["exact-64", "exact-128", "uneven", "12-per-key"])
@pytest.mark.parametrize("sizes", [[1000], [90]])
def test_attention_long_prompts(run, name, sizes):
    """Portions of several row blocks, with earlier keys before them."""
    dev, dtype = run
    if dev.type == "cpu":
        pytest.skip("the CPU implementation has one form")
    sh, m = _shape(name)
    w = _norms(sh)
    qkvs = [rnd(n, sh.width, seed=60 + n).to(dtype).double() for n in (210, 141)]
    got = _run_heads(sh, qkvs, w, sizes, dev, dtype, block_size=64)
    for g, x in zip(got, qkvs):
        close(g, _oracle_heads(sh, m, x, w), dtype, bf16=2e-2)


@pytest.mark.parametrize("name", ["odd", "exact-64", "uneven", "window-1", "exact-80"])
@pytest.mark.parametrize("mode", ["prompt", "decode", "short-blocks"])
def test_one_loud_key_at_every_distance(run, name, mode):
    """One key's score towers over all others and the sink; queries at every distance from it see exactly it, or do
    not."""
    dev, dtype = run
    sh, m = _shape(name, gated=False)
    if mode == "short-blocks" and not (dev.type == "cuda" and head_blocks_ok(sh, dtype)):
        pytest.skip("no block form here")
    n, bs = 70, 8
    w = {"q.norm": None, "k.norm": None, "sink": torch.zeros(sh.heads).double()}
    for loud in (0, 7, 8, 15, 31, 33):
        x = torch.zeros(n, sh.width, dtype=torch.float64)
        q, k, v = x.split([sh.heads * sh.dim, sh.kv_heads * sh.dim, sh.kv_heads * sh.vdim], 1)
        q.view(n, sh.heads, sh.dim)[:, :, 0] = 8.0 / sh.scale
        v[:] = rnd(n, v.shape[1], seed=loud)
        k.view(n, sh.kv_heads, sh.dim)[loud, :, 0] = 4.0
        x = x.to(dtype).double()
        sizes = {"prompt": [n], "decode": [1], "short-blocks": [2]}[mode]
        (got, ) = _run_heads(sh, [x], w, sizes, dev, dtype, block_size=bs, decode_max=0 if mode == "short-blocks" else None)
        value = v[loud].to(dtype).double().view(sh.kv_heads, sh.vdim).repeat_interleave(sh.heads // sh.kv_heads, 0)
        value = value.reshape(-1)
        win = sh.window or 10**9
        for i in range(n):
            same = float((got[i] - value).norm() / value.norm())
            assert (same < 0.05) == (0 <= i - loud < win), (loud, i, same)


@pytest.mark.parametrize("name", ["odd", "exact-64", "12-per-key"])
@pytest.mark.parametrize("sizes", [[1000], [1]])
def test_sink_and_gate(run, name, sizes):
    """A sink far above the scores silences its head, one far below is as none; a closed gate silences its head."""
    dev, dtype = run
    sh, m = _shape(name)
    w = _norms(sh)
    n = 24
    x = rnd(n, sh.width, seed=3).to(dtype).double()
    x[:, sh.qkv_width:] = 0.0
    head = lambda t, h: t[:, h * sh.vdim:(h + 1) * sh.vdim]  # noqa: E731
    w["sink"] = torch.full((sh.heads, ), -80.0).double()
    w["sink"][1] = 80.0
    (a, ) = _run_heads(sh, [x], w, sizes, dev, dtype)
    (b, ) = _run_heads(sh, [x], dict(w, sink=None), sizes, dev, dtype)
    assert head(a, 1).abs().max() < 1e-6 < head(b, 1).abs().max()
    close(head(a, 0), head(b, 0), dtype, f32=1e-6, bf16=1e-6)
    # the first token sees itself and the sink: its value times e^s / (e^s + e^sink) times the gate
    w["sink"] = torch.full((sh.heads, ), 1.3).double()
    x[:, sh.qkv_width + 2] = -60.0
    (c, ) = _run_heads(sh, [x], w, sizes, dev, dtype)
    want = _oracle_heads(sh, m, x, w)
    close(c[:1], want[:1], dtype, bf16=2e-2)
    assert head(c, 2).abs().max() < 1e-6


def test_attention_without_norms_and_gate(run):
    dev, dtype = run
    sh, m = _shape("uneven", gated=False)
    w = {"q.norm": None, "k.norm": None, "sink": None}
    x = rnd(30, sh.width, seed=5, scale=0.7).to(dtype).double()
    (got, ) = _run_heads(sh, [x], w, [13, 1, 9], dev, dtype)
    H, G, d, vd = sh.heads, sh.kv_heads, sh.dim, sh.vdim
    q, k, v = x[:, :H * d].view(-1, H, d), x[:, H * d:(H + G) * d].view(-1, G, d), x[:, (H + G) * d:].view(-1, G, vd)
    want = torch.zeros(30, H, vd, dtype=torch.float64)
    for i in range(30):
        for h in range(H):
            s = torch.softmax(k[:i + 1, h // (H // G)] @ q[i, h] * sh.scale, 0)
            want[i, h] = s @ v[:i + 1, h // (H // G)]
    close(got, want.view(30, -1), dtype, bf16=2e-2)


# -----------------------------------------------------------------------------------------------
# norms
# -----------------------------------------------------------------------------------------------
@pytest.mark.parametrize("T,W,pad", [(5, 64, 128), (1, 37, 8), (3, 2048, 128), (1030, 72, 128), (2, 4104, 1),
                                     (1025, 1536, 128), (1, 9000, 8)])
def test_residual_norm(run, T, W, pad):
    dev, dtype = run
    if dev.type == "cpu" and T * W > 10**6:
        pytest.skip("large")
    x, d = rnd(T, W, seed=1, scale=3.0).float().double(), rnd(T, W, seed=2, scale=0.1).to(dtype).double()
    g = (1 + 0.5 * rnd(W, seed=3)).float().double()
    x1, rows = residual_norm(x.float().to(dev), d.to(dtype).to(dev), g.float().to(dev), 1e-3, dtype, pad)
    want = x + oracle.rms(d, 1e-3, g)
    close(x1, want, torch.float32)
    close(rows[:, :W], want, dtype, bf16=5e-3)
    assert (rows[:, W:] == 0).all() and rows.shape[1] % pad == 0 and rows.dtype == dtype


def test_embedding_and_output_norm(run):
    dev, dtype = run
    for W in (48, 50):
        emb = rnd(11, W, seed=1).to(dtype)
        ids = torch.tensor([3, 0, 10, 3])
        x, rows = embed_rows(emb.to(dev), ids.to(dev), 2.5, dtype, 32)
        close(x, emb.double()[ids] * 2.5, torch.float32, f32=1e-6)
        close(rows[:, :W], emb.double()[ids] * 2.5, dtype, bf16=5e-3)
        assert (rows[:, W:] == 0).all() and rows.shape[1] == 64
        g = 1 + rnd(W, seed=2)
        got = norm_rows(x, None, torch.tensor([2, 0], dtype=torch.int32, device=dev), g.float().to(dev), 1e-2, dtype)
        close(got, oracle.rms(emb.double()[ids[[2, 0]]] * 2.5, 1e-2, g), dtype, bf16=5e-3)


# -----------------------------------------------------------------------------------------------
# router and experts
# -----------------------------------------------------------------------------------------------
ROUTERS = {"plain": RouterShape(6, 0, 2, 1, 1, 1.0), "identity": RouterShape(7, 2, 3, 1, 1, 2.5),
           "groups": RouterShape(11, 4, 4, 5, 2, 0.7), "all": RouterShape(3, 1, 4, 1, 1, 1.0),
           "one": RouterShape(1, 0, 1, 1, 1, 3.0), "keep-all": RouterShape(12, 0, 5, 4, 4, 1.0),
           "many": RouterShape(150, 30, 8, 9, 3, 1.5), "more": RouterShape(700, 20, 3, 36, 10, 1.0)}


def _cfg(r, ff, shared=0):
    return {"router": {"experts": r.experts, "identity": r.identity, "top": r.top, "scale": r.scale,
                       "groups": {"count": r.groups, "keep": r.keep}}, "expert": {"ff": ff},
            "shared": {"ff": shared} if shared else None}


@pytest.mark.parametrize("name", list(ROUTERS))
def test_route(run, name):
    dev, _ = run
    r, T = ROUTERS[name], 37
    z = rnd(T, r.outputs + 1, seed=1, scale=1.5).float()
    # corrections of both signs, as large as the scores: they decide, groups hold negative choice scores
    c = (rnd(r.outputs, seed=2) * 0.4).float()
    e, w = route(z.to(dev), c.to(dev), r)
    for t in range(T):
        chosen, weights = oracle.route(z[t, :r.outputs].double(), c.double(), _cfg(r, 1)["router"])
        got = dict(zip(e[t].tolist(), w[t].tolist()))
        assert set(got) == set(chosen) and len(got) == r.top
        for i, v in zip(chosen, weights):
            assert abs(got[i] - float(v)) < 1e-5 * max(1.0, r.scale)


def test_group_of_negative_choices_is_not_outranked_by_a_dropped_one(run):
    """All choice scores of the kept group are negative: the experts of the dropped group stay out all the same."""
    dev, _ = run
    r = RouterShape(4, 0, 2, 2, 1, 1.0)
    z = torch.zeros(1, 4)
    c = torch.tensor([-0.3, -5.0, -0.6, -0.61])
    e, w = route(z.to(dev), c.to(dev), r)
    assert sorted(e[0].tolist()) == [0, 1]
    assert torch.allclose(w.cpu(), torch.full((1, 2), 0.25))


def _expert_weights(r, W, ff, shared, seed=0, router=1.0):
    p = {"router": rnd(r.outputs, W, seed=seed + 1, scale=router * W**-0.5),
         "correction": rnd(r.outputs, seed=seed + 2, scale=0.1)}
    for e in range(r.experts):
        p[f"e{e}.gate"] = rnd(ff, W, seed=seed + 10 + e, scale=W**-0.5)
        p[f"e{e}.up"] = rnd(ff, W, seed=seed + 1000 + e, scale=W**-0.5)
        p[f"e{e}.down"] = rnd(W, ff, seed=seed + 2000 + e, scale=ff**-0.5)
    if shared:
        p["shared.gate"] = rnd(shared, W, seed=seed + 3, scale=W**-0.5)
        p["shared.up"] = rnd(shared, W, seed=seed + 4, scale=W**-0.5)
        p["shared.down"] = rnd(W, shared, seed=seed + 5, scale=shared**-0.5)
        p["shared.sg"] = rnd(1, W, seed=seed + 6, scale=W**-0.5)
    return {k: v.to(torch.bfloat16).double() for k, v in p.items()}


def _layer(r, W, ff, shared, p, dev, dtype):
    """The registered module and its weights on the device."""
    mod = instantiate_expert_layer(DSExpertLayerConfig(W, ff, r, shared, 1, dtype))
    st = {k: torch.stack([p[f"e{e}.{k}"] for e in range(r.experts)]) for k in ("gate", "up", "down")}
    st.update({k: v for k, v in p.items() if not re.match(r"e\d", k)})
    w = mod.shard(st, lambda t: t, lambda t: t)
    return mod, {k: None if v is None else (v.float() if k == "router.c" else v.to(dtype)).contiguous().to(dev)
                 for k, v in w.items()}


EXPERTS = {"small": (ROUTERS["plain"], 48, 24, 40), "identity": (ROUTERS["identity"], 72, 40, 16),
           "groups": (ROUTERS["groups"], 136, 56, 0), "odd": (ROUTERS["one"], 37, 11, 5),
           "all": (ROUTERS["all"], 200, 136, 264), "tile": (ROUTERS["plain"], 256, 128, 128)}


@pytest.mark.parametrize("name", list(EXPERTS))
@pytest.mark.parametrize("T", [1, 3, 20, 64, 65, 200])
@pytest.mark.parametrize("form", ["default", "sorted"])
def test_expert_layer(run, name, T, form, monkeypatch):
    """Product by product against the oracle, which is handed the choices (their own test is test_route)."""
    dev, dtype = run
    if form == "sorted":
        if dev.type == "cpu" or dtype == torch.float32 or T > 64:
            pytest.skip("the default form here")
        monkeypatch.setattr(experts_op, "SKINNY_TOKENS", 0)
    r, W, ff, shared = EXPERTS[name]
    p = _expert_weights(r, W, ff, shared)
    mod, w = _layer(r, W, ff, shared, p, dev, dtype)
    x = rnd(T, W, seed=9).to(dtype)
    rows = torch.zeros(T, w["w13"].shape[2], dtype=dtype, device=dev)
    rows[:, :W] = x.to(dev)
    x32 = x.float().to(dev)
    parts = mod(rows, w)
    h = x.double()
    want = torch.zeros(T, W, dtype=torch.float64)
    for t in range(T):
        s = torch.softmax(p["router"] @ h[t], 0)
        for e in parts.expert[t].tolist():
            y = h[t] if e >= r.experts else oracle.expert(h[t], p[f"e{e}.gate"], p[f"e{e}.up"], p[f"e{e}.down"])
            want[t] += s[e] * r.scale * y
        if dtype == torch.float32:
            assert set(parts.expert[t].tolist()) == set(oracle.route(p["router"] @ h[t], p["correction"],
                                                                      _cfg(r, ff)["router"])[0])
    if shared:
        sg = torch.sigmoid(h @ p["shared.sg"].T)
        want += sg * oracle.expert(h, p["shared.gate"], p["shared.up"], p["shared.down"])
    close(sum_experts(x32, parts, dtype), want, dtype, bf16=2e-2)
    g = 1 + 0.2 * rnd(W, seed=12)
    x1, _ = residual_norm(x32.clone(), parts, g.float().to(dev), 1e-4, dtype, 1)
    close(x1, h + oracle.rms(want, 1e-4, g), dtype, f32=2e-5, bf16=2e-2)
    if dtype == torch.float32 and r.identity:  # left to another rank
        parts.identity = False
        got = sum_experts(x32, parts, dtype).double().cpu()
        for t in range(T):
            s = torch.softmax(p["router"] @ h[t], 0)
            want[t] -= sum(s[e] * r.scale for e in parts.expert[t].tolist() if e >= r.experts) * h[t]
        close(got, want, dtype)


@GPU
@pytest.mark.parametrize("T,E,k,W,ff", [(700, 2, 2, 256, 256), (1300, 3, 1, 512, 384), (300, 5, 3, 384, 128)])
def test_sorted_products_of_every_tile(T, E, k, W, ff):
    """Long steps: 256-row tiles where the experts are full enough, else 128-row tiles."""
    dev, dtype = torch.device("cuda"), torch.bfloat16
    print(f"T={T} E={E} k={k} W={W} ff={ff}", flush=True)
    r = RouterShape(E, 0, k, 1, 1, 1.0)
    p = _expert_weights(r, W, ff, 0)
    mod, w = _layer(r, W, ff, 0, p, dev, dtype)
    x = rnd(T, W, seed=9).to(dtype)
    parts = mod(x.to(dev), w)
    h = x.double()
    s = torch.softmax(h @ p["router"].T, -1)
    on = torch.zeros(T, E, dtype=torch.float64).scatter_(1, parts.expert.long().cpu(), 1.0)
    want = sum((s * on)[:, e:e + 1] * oracle.expert(h, p[f"e{e}.gate"], p[f"e{e}.up"], p[f"e{e}.down"])
               for e in range(E))
    close(sum_experts(x.float().to(dev), parts, dtype), want, dtype, bf16=2e-2)


# -----------------------------------------------------------------------------------------------
# models
# -----------------------------------------------------------------------------------------------
def _att(heads, kv, dim, vdim, window, mlp):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
                                           "scale": 1.3 * dim**-0.5, "mask": {"size": window}}, "mlp": mlp}


def _moe(r, ff, shared):
    return dict(_cfg(r, ff, shared), kind="moe")


_A = _att(4, 2, 16, 24, 9, _moe(RouterShape(5, 1, 2, 3, 2, 1.5), 24, 40))
_B = _att(3, 3, 32, 32, 33, None)
_C = _att(6, 1, 24, 16, 70, _moe(RouterShape(4, 0, 3, 1, 1, 1.0), 40, 0))
_D = _att(1, 1, 8, 8, 1, _moe(RouterShape(3, 3, 2, 2, 1, 2.0), 16, 8))
_E = _att(8, 1, 128, 128, 100, _moe(RouterShape(8, 0, 1, 4, 3, 1.0), 136, 64))
_O = _att(3, 1, 5, 7, 12, _moe(RouterShape(3, 2, 2, 5, 3, 1.7), 11, 9))
CONFIGS = {
    # layers of different sizes, some without feed-forward, weights used again near and far, forwards in the list too
    "mixed": dict(vocab=131, width=64, norm={"eps": 1e-5}, embedding={"scale": 6.0}, logit_scale=1.5,
                  layers=[_A, _B, dict(_A, weights_of=0), _C, dict(_B, weights_of=1), _D]),
    "later": dict(vocab=90, width=40, norm={"eps": 1e-4}, embedding={"scale": 5.5}, logit_scale=0.7,
                  layers=[dict(_D, weights_of=2), _C, _D, dict(_D, weights_of=0)]),
    "wide": dict(vocab=67, width=72, norm={"eps": 1e-6}, embedding={"scale": 5.0}, logit_scale=1.0, layers=[_E]),
    # sizes the matrix-core and vector paths do not take
    "odd": dict(vocab=61, width=37, norm={"eps": 1e-6}, embedding={"scale": 5.0}, logit_scale=2.2,
                layers=[_O, dict(_O, weights_of=0)]),
}
ALPHA = 0.2  # router gain


def _choice_margin(z, correction, r):
    """How far the nearest other choice is, in score, for one token."""
    c = torch.softmax(z, -1) + correction
    n, size = c.numel(), c.numel() // r["groups"]["count"]
    best, _ = c.view(-1, size).max(-1)
    top = best.sort(descending=True).values
    keep = r["groups"]["keep"]
    m = float("inf") if keep == top.numel() else float(top[keep - 1] - top[keep])
    kept = best.topk(keep).indices
    a = torch.cat([c[g * size:(g + 1) * size] for g in kept]).sort(descending=True).values
    return m if r["top"] == a.numel() else min(m, float(a[r["top"] - 1] - a[r["top"]]))


def make_weights(cfg, seed=0):
    """Random weights, rounded to bfloat16 values. Queries and keys are loud enough that single keys matter. Rounding must
    not decide which expert runs (the logits would jump), so each token's embedding carries a code of well separated
    strengths along directions that all routers read, chosen such that no router is near a tie on it."""
    g = torch.Generator().manual_seed(seed)
    w, W, V = {}, cfg["width"], cfg["vocab"]

    def lin(name, rows, cols, scale=1.0):
        w[name] = torch.randn(rows, cols, generator=g) * scale * cols**-0.5

    owners = [(i, e) for i, e in enumerate(cfg["layers"]) if e.get("weights_of") is None]
    routed = [(i, e["mlp"]["router"]) for i, e in owners if e["mlp"]]
    n_of = {i: r["experts"] + r["identity"] for i, r in routed}
    n_dir = max(n_of.values())
    U = torch.linalg.qr(torch.randn(W, n_dir, generator=g))[0].T
    perm = {i: torch.randperm(n_dir, generator=g)[:n] for i, n in n_of.items()}
    corr = {i: torch.randn(n, generator=g) * 0.15 for i, n in n_of.items()}
    embed = []
    for _ in range(V):
        for _ in range(2000):
            code = torch.randperm(n_dir, generator=g).float() - n_dir / 2
            z = {i: ALPHA * cfg["embedding"]["scale"] * code[perm[i]] for i in n_of}
            if all(_choice_margin(z[i], corr[i], r) > 0.06 for i, r in routed):
                break
        else:
            raise AssertionError("no code is clear for every router")
        rest = torch.randn(W, generator=g)
        embed.append(code @ U + rest - (U @ rest) @ U)
    w["embed"] = torch.stack(embed)
    for i, e in owners:
        p, m = f"l{i}.", e["mixer"]
        H, G = m["heads"], m["kv_heads"]
        lin(p + "mix.q", H * m["dim"], W)
        lin(p + "mix.k", G * m["dim"], W)
        lin(p + "mix.v", G * m["vdim"], W)
        lin(p + "mix.g", H, W)
        lin(p + "mix.o", W, H * m["vdim"])
        w[p + "mix.q.norm"] = 1.5 + 0.3 * torch.randn(m["dim"], generator=g)
        w[p + "mix.k.norm"] = 1.5 + 0.3 * torch.randn(m["dim"], generator=g)
        w[p + "mix.sink"] = torch.randn(H, generator=g)
        w[p + "norm1"] = -0.75 + 0.08 * torch.randn(W, generator=g)
        if e["mlp"]:
            w[p + "norm2"] = -0.75 + 0.08 * torch.randn(W, generator=g)
            ff, sh = e["mlp"]["expert"]["ff"], e["mlp"]["shared"]
            w[p + "mlp.router"], w[p + "mlp.correction"] = ALPHA * U[perm[i]], corr[i]
            for x in range(e["mlp"]["router"]["experts"]):
                lin(f"{p}mlp.e{x}.gate", ff, W)
                lin(f"{p}mlp.e{x}.up", ff, W)
                lin(f"{p}mlp.e{x}.down", W, ff)
            if sh:
                lin(p + "mlp.shared.gate", sh["ff"], W)
                lin(p + "mlp.shared.up", sh["ff"], W)
                lin(p + "mlp.shared.down", W, sh["ff"])
                lin(p + "mlp.shared.sg", 1, W)
    w["final.norm"] = 0.2 * torch.randn(W, generator=g)
    lin("head", V, W)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


_CACHE = {}


def model(name):
    if name not in _CACHE:
        cfg = dict(CONFIGS[name], architecture="Buvuzen")
        _CACHE[name] = (cfg, make_weights(cfg))
    return _CACHE[name]


def oracle_logits(name, toks):
    key = (name, tuple(toks))
    if key not in _CACHE:
        cfg, w = model(name)
        margins = []
        plain = oracle.route

        def watched(z, correction, r):
            margins.append(_choice_margin(z, correction, r))
            return plain(z, correction, r)

        oracle.route = watched
        try:
            _CACHE[key] = oracle.forward(cfg, {k: v.double() for k, v in w.items()}, list(toks))[0]
        finally:
            oracle.route = plain
        # no choice of an expert is near a tie on this sequence, so rounding cannot change it
        assert min(margins) > 0.002, (name, min(margins))
    return _CACHE[key]


def engine(name, run, blocks=12, slots=4, block_size=16, max_context=192, **conf):
    dev, dtype = run
    cfg, w = model(name)
    spec = spec_from_hf(cfg)
    ec = RaggedInferenceEngineConfig.from_dict(dict(
        dtype="fp32" if dtype == torch.float32 else "bf16",
        state_manager=dict(max_context=max_context, max_ragged_batch_size=512, max_tracked_sequences=slots,
                           kv_block_size=block_size), **conf))
    return InferenceEngineV2(spec, convert_hf(w, spec), ec, device=dev, num_kv_blocks=blocks)


def tokens_of(name, n, seed):
    return tokens(CONFIGS[name]["vocab"], n, seed)


def check_logits(got, want, dtype, bf16=6e-2):
    close(got, want, dtype, f32=1e-4, bf16=bf16)


@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("sizes", [[1000], [2], [1], [21, 1, 16, 2, 3, 17]])
def test_portions(run, name, sizes):
    """Whole prompts, portions of several sizes and single tokens give the logits of the whole sequence."""
    eng = engine(name, run)
    toks = tokens_of(name, 61, 1)
    got, = feed(eng, [toks], portions([61], sizes))
    check_logits(got, oracle_logits(name, toks), run[1])
    eng.flush(0)
    assert eng.free_blocks == 12


@pytest.mark.parametrize("name", list(CONFIGS))
def test_mixed_batches(run, name):
    """Unequal requests, portions beside single tokens: each gets the logits it gets alone."""
    seqs = [tokens_of(name, n, 10 + n) for n in (50, 1, 23, 37)]
    got = feed(engine(name, run, blocks=16), seqs, portions([len(s) for s in seqs], [19, 1, 1, 2, 30, 1, 5], seed=3))
    for g, s in zip(got, seqs):
        check_logits(g, oracle_logits(name, s), run[1])


def test_long_mixed_step(run):
    """A step of more tokens than the direct expert products take, single tokens of other requests beside it."""
    seqs = [tokens_of("mixed", n, 70 + n) for n in (130, 9, 12)]
    steps = [[(1, 8, 0), (2, 11, 0)], [(0, 100, 0), (1, 1, 8), (2, 1, 11)], [(0, 30, 100)]]
    got = feed(engine("mixed", run, blocks=16), seqs, steps)
    for g, s in zip(got, seqs):
        check_logits(g, oracle_logits("mixed", s), run[1])


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_pages_and_slots_are_used_again(run, name):
    eng = engine(name, run, blocks=8, slots=2)
    first = feed(eng, [tokens_of(name, 60, 20), tokens_of(name, 60, 21)], [[(0, 60, 0), (1, 60, 0)]])
    assert eng.free_blocks == 0
    with pytest.raises(SchedulingError):
        eng.put([7], [torch.tensor([1])], capture_latents=False)
    eng.flush(0)
    s = tokens_of(name, 33, 22)
    outs = []
    for p, n in ((0, 20), (20, 1), (21, 1), (22, 11)):
        lg, _ = eng.put([5], [torch.tensor(s[p:p + n])], capture_latents=False, logits_at=[range(n)])
        outs.append(lg.double().cpu())
    check_logits(torch.cat(outs), oracle_logits(name, s), run[1])
    check_logits(first[1], oracle_logits(name, tokens_of(name, 60, 21)), run[1])
    eng.flush(5)
    lg, _ = eng.put([9], [torch.tensor(s[:1])], capture_latents=False)  # one token on pages full of old rows
    check_logits(lg, oracle_logits(name, s)[:1], run[1])


def test_long_decoding(run):
    """Many single tokens, past every window, across pages; the batch's other sequence is at another position."""
    toks, other = tokens_of("mixed", 130, 30), tokens_of("mixed", 120, 31)
    steps = [[(0, 5, 0)], [(1, 2, 0)]] + [[(0, 1, 5 + i)] + ([(1, 1, 2 + i)] if i < 118 else []) for i in range(125)]
    got = feed(engine("mixed", run, blocks=24), [toks, other], steps)
    check_logits(got[0], oracle_logits("mixed", toks), run[1])
    check_logits(got[1], oracle_logits("mixed", other), run[1])


def test_wanted_places(run):
    eng = engine("mixed", run)
    a, b = tokens_of("mixed", 30, 1), tokens_of("mixed", 12, 2)
    lg, _ = eng.put(["a", "b"], [torch.tensor(a), torch.tensor(b)], capture_latents=False, logits_at=[[4, 29, 0], []])
    check_logits(lg, oracle_logits("mixed", a)[[4, 29, 0]], run[1])
    lg, _ = eng.put(["b"], [torch.tensor(b[:1])], capture_latents=False, logits_at=[[]])
    assert lg.shape == (0, 131)


def test_shared_weights_have_caches_of_their_own(run):
    """A layer that uses another layer's weights attends to its own keys: one cached row width per run, and evicting and
    restoring every run's rows gives the same logits again (HCache latents are the cached rows)."""
    eng = engine("mixed", run, blocks=8)
    m = eng.model()
    assert len(m.layers) == 4 and len(m.runs) == 6 and run_order(m.spec) == [0, 1, 0, 2, 1, 3]
    assert m.row_widths == [2 * 40, 3 * 64, 2 * 40, 40, 3 * 64, 16] and m.state_floats() == 0
    s, o = tokens_of("mixed", 40, 3), tokens_of("mixed", 25, 4)
    lats = []
    for p, n in ((0, 22), (22, 1), (23, 1), (24, 9)):
        lg, (lat, ) = eng.put([1], [torch.tensor(s[p:p + n])])
        lats.append(lat.clone())
    assert lats[0].shape == (1, 22, sum(m.row_widths))
    eng.evict(1)
    feed(eng, [o], [[(0, 25, 0)]])  # other rows in the freed pages
    eng.restore_kv([1], [torch.tensor(s[:33])], [torch.cat(lats, 1)])
    got = [eng.put([1], [torch.tensor(s[33 + i:34 + i])], capture_latents=False)[0].double().cpu() for i in range(7)]
    check_logits(torch.cat(got), oracle_logits("mixed", s)[33:], run[1])


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_greedy_generation(run, name):
    """The engine's own generation loop; compared with the plain implementation step by step along its own tokens."""
    prompt = tokens_of(name, 19, 5)
    eng = engine(name, run, blocks=8)
    out = eng.generate(1, torch.tensor(prompt), max_new_tokens=24)
    lg = oracle_logits(name, prompt + out)[len(prompt) - 1:-1]
    picked = lg[torch.arange(24), out]
    assert ((lg.max(-1).values - picked) <= (1e-4 if run[1] == torch.float32 else 0.25)).all()
    if run[1] == torch.float32:
        assert out == lg.argmax(-1).tolist()
    eng.flush(1)
    g = torch.Generator(device=run[0]).manual_seed(0)
    sampled = eng.generate(2, torch.tensor(prompt), max_new_tokens=8, do_sample=True, temperature=0.7, top_k=5,
                           generator=g)
    lg = oracle_logits(name, prompt + sampled)[len(prompt) - 1:-1]
    rank = (lg > lg[torch.arange(8), sampled][:, None]).sum(-1)
    assert (rank <= (4 if run[1] == torch.float32 else 12)).all()


@GPU
@pytest.mark.parametrize("B", [1, 2, 5, 20])
@pytest.mark.parametrize("capture", [False, True])
def test_decode_graph_replays(B, capture):
    """Captured decode steps against the eager ones over several replays with eager work and other requests between
    them, and captured latents are the cached rows."""
    run = (torch.device("cuda"), torch.bfloat16)
    print(f"graph B={B} capture={capture}", flush=True)
    seqs = [tokens_of("mixed", 30, 100 + s) for s in range(B)]
    outs, lats = {}, {}
    for graph in (True, False):
        eng = engine("mixed", run, blocks=3 * B + 4, slots=B + 1)
        if not graph:
            eng.model().decode_graph_max_batch = 0
        eng.put(list(range(B)), [torch.tensor(s[:11 + i % 3]) for i, s in enumerate(seqs)], capture_latents=False)
        o, la = [], []
        for k in range(6):
            if k == 3:
                eng.put(["x"], [torch.tensor(seqs[0][:7])], capture_latents=False)
                torch.cuda.synchronize()
                eng.flush("x")
            lg, lat = eng.put(list(range(B)), [torch.tensor(s[11 + i % 3 + k:12 + i % 3 + k])
                                               for i, s in enumerate(seqs)], capture_latents=capture)
            o.append(lg.double().cpu())
            if capture:
                la.append(torch.cat([x.double() for x in lat], 1).clone())
        outs[graph] = torch.stack(o)
        lats[graph] = la
        assert bool(eng.model()._decode_graphs) == graph
    assert torch.equal(outs[True], outs[False])
    for a, b in zip(lats[True], lats[False]):
        assert torch.equal(a, b)
    for i, s in enumerate(seqs[:3]):
        check_logits(outs[True][:, i], oracle_logits("mixed", s)[11 + i % 3:17 + i % 3], torch.bfloat16)


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_serialize_and_reload(run, name, tmp_path):
    eng = engine(name, run)
    s = tokens_of(name, 20, 6)
    a, = feed(eng, [s], [[(0, 20, 0)]])
    eng.serialize(str(tmp_path))
    conf = {"dtype": "fp32" if run[1] == torch.float32 else "bf16",
            "state_manager": {"max_context": 192, "kv_block_size": 16, "max_tracked_sequences": 2}}
    eng2 = build_engine_from_ds_checkpoint(str(tmp_path), conf, device=run[0], num_kv_blocks=4)
    b, = feed(eng2, [s], [[(0, 20, 0)]])
    assert torch.equal(a, b)


def test_weight_only_quantization():
    eng = engine("mixed", (torch.device("cpu"), torch.float32), quantization={"quantization_mode": "int8"})
    s = tokens_of("mixed", 20, 6)
    got, = feed(eng, [s], [[(0, 13, 0)], [(0, 7, 13)]])
    close(got, oracle_logits("mixed", s), torch.float32, f32=0.1)


def _tp_config():
    r = RouterShape(3, 2, 3, 5, 4, 1.5)
    a = _att(4, 2, 16, 24, 9, _moe(r, 24, 40))
    b = _att(6, 6, 8, 16, 33, None)
    return dict(CONFIGS["mixed"], architecture="Buvuzen", layers=[a, b, dict(a, weights_of=0)])


def _tp_worker(rank, world, path):
    import hcache_deepspeed_amd as hds
    hds.init_distributed(dist_backend="gloo", verbose=False)
    cfg = _tp_config()
    w = make_weights(cfg)
    spec = spec_from_hf(cfg)
    ec = RaggedInferenceEngineConfig.from_dict(dict(
        dtype="fp32", tensor_parallel={"tp_size": world},
        state_manager=dict(max_context=64, kv_block_size=16, max_tracked_sequences=2)))
    eng = InferenceEngineV2(spec, convert_hf(w, spec), ec, device=torch.device("cpu"), num_kv_blocks=4)
    s = tokens_of("mixed", 24, 8)
    got, = feed(eng, [s], [[(0, 17, 0)], [(0, 1, 17)], [(0, 6, 18)]])
    check_logits(got, oracle.forward(cfg, {k: v.double() for k, v in w.items()}, s)[0], torch.float32)


def test_tensor_parallel_gloo():
    from .dist_utils import run_distributed
    run_distributed(_tp_worker, 2, None)


def test_trace_replay(run, tmp_path):
    """The trace runner's step function and the checkpoint folder it reads."""
    from safetensors.torch import save_file

    from hcache_deepspeed_amd.inference.v2 import trace
    cfg, w = model("mixed")
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    eng = trace.build_engine(str(tmp_path), "float32" if run[1] == torch.float32 else "bfloat16", 192, device=run[0])
    a, b = tokens_of("mixed", 40, 1), tokens_of("mixed", 70, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:30], "want": [0, 7]},
                                     {"id": "b", "tokens": b[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[2:70], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": [3], "want": [0]},
                                     {"id": "a", "tokens": a[30:31], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "c", "tokens": a[:1], "want": [0]}], "end": ["b", "c"]}]
    for st in steps:
        trace.run_step(eng, st, str(tmp_path))
    assert not (tmp_path / "1.f32").exists() and eng.free_blocks == 3

    def read(k):
        return torch.frombuffer(bytearray((tmp_path / f"{k}.f32").read_bytes()), dtype=torch.float32).view(-1, 131)

    check_logits(read(0), oracle_logits("mixed", a)[[0, 7]], run[1])
    want = torch.stack([oracle_logits("mixed", b + [3])[70], oracle_logits("mixed", a)[30]])
    check_logits(read(2), want, run[1])
    check_logits(read(3), oracle_logits("mixed", a)[:1], run[1])


def test_kernel_sources_of_the_model_class_are_complete():
    """A library of the class's KERNEL_SOURCES alone exports every entry point its ops call."""
    from hcache_deepspeed_amd.ops import build, gemv, output_norm, paged
    cls = transformer_class(spec_from_hf(model("mixed")[0]))
    have = ""
    for f in cls.KERNEL_SOURCES:
        with open(os.path.join(build.CSRC, "kernels", f)) as fh:
            have += fh.read()
    used = {"hds_glu_rows"}
    for mod in (gemv, experts_op, output_norm, paged):
        with open(mod.__file__) as fh:
            used |= set(re.findall(r"\)?\.(hds_\w+)\(", fh.read()))
    assert len(used) > 20
    for name in used - {"hds_gemv_recur_bf16"}:
        assert re.search(rf"HDS_EXPORT int {name}\(", have), name


def test_checkpoint_folder_and_registry(tmp_path):
    from safetensors.torch import save_file
    cfg, w = model("later")
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    eng = build_hf_engine(str(tmp_path), {"dtype": "fp32", "state_manager": {"max_context": 64}},
                          device=torch.device("cpu"), num_kv_blocks=4)
    assert run_order(eng.model().spec) == [0, 1, 0, 0] and len(eng.model().row_widths) == 4
    s = tokens_of("later", 9, 1)
    lg, _ = eng.put([1], [torch.tensor(s)])
    check_logits(lg, oracle_logits("later", s)[-1:], torch.float32)
    for bad in (dict(cfg["layers"][1], type="other"), dict(cfg["layers"][1], mlp={"kind": "other"})):
        with pytest.raises(NotImplementedError):
            spec_from_hf(dict(cfg, layers=[bad]))
    with pytest.raises(ValueError):
        spec_from_hf(dict(cfg, layers=[dict(cfg["layers"][1], weights_of=0)]))
    with pytest.raises(NotImplementedError):
        RouterShape(1500, 0, 2).check()
    with pytest.raises(NotImplementedError):
        RouterShape(6, 0, 3, 3, 1).check()
