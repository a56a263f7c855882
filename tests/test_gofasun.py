"""Gofasun on the ragged serving engine against the plain implementation in gofasun_oracle.py: every mechanism alone,
then the engine with whole prompts, portions, single tokens, mixed batches, reused pages and slots, decode graphs,
eviction, tensor parallelism, serialization, generation and trace replay. CPU runs use the ops' torch implementations,
``gpu`` runs the HIP kernels in 32-bit and in bfloat16."""
import json
import math

import pytest
import torch

from hcache_deepspeed_amd.inference.v2 import build_engine_from_ds_checkpoint, build_hf_engine
from hcache_deepspeed_amd.inference.v2.arch import convert_hf, spec_from_hf
from hcache_deepspeed_amd.inference.v2.engine import InferenceEngineV2, RaggedInferenceEngineConfig, SchedulingError
from hcache_deepspeed_amd.ops.activations import glu_rows
from hcache_deepspeed_amd.ops.gated_scan import gated_scan, recur_step
from hcache_deepspeed_amd.ops.gemv import glu_gemv
from hcache_deepspeed_amd.ops.input_norm import input_norm, norm_rows
from hcache_deepspeed_amd.ops.latent_attention import LatentShape, can_expand, latent_attention, make_plan
from hcache_deepspeed_amd.ops.rope import rope_tables

from . import gofasun_oracle as oracle
from .serving_utils import GPU, Pages, close, feed, portions, rnd, run, tokens  # noqa: F401

# -----------------------------------------------------------------------------------------------
# mechanisms
# -----------------------------------------------------------------------------------------------
@pytest.mark.parametrize("W,taps,two,vector", [(64, 3, True, False), (37, 2, True, True), (40, 1, False, False),
                                               (96, 4, True, False), (20, 6, False, True), (28, 12, True, False)])
@pytest.mark.parametrize("sizes", [[1000], [1], [2], [17, 1, 5, 2, 40]])
def test_input_norm(run, W, taps, two, vector, sizes):
    dev, dtype = run
    eps, lengths, slots = 1e-3, [50, 3, 1, 33], [3, 0, 2, 1]
    k = 2 if two else 1
    gains = [rnd(W if vector else 1, seed=1 + i) + 1 for i in range(k)]
    convs = [rnd(taps, W, seed=3 + i) for i in range(k)]
    pages = Pages(4, 4, 64, 8, slots, dev, dtype)
    state = torch.full((4, 8 + (taps - 1) * W + (-(taps - 1) * W) % 4), 7.0, device=dev)  # stale slots
    xs = [rnd(n, W, seed=10 + s).float().double() for s, n in enumerate(lengths)]
    ds = [rnd(n, W, seed=20 + s).to(dtype).double() for s, n in enumerate(lengths)]
    ys = [[[] for _ in range(k)] for _ in lengths]
    for step in portions(lengths, sizes):
        b = pages.batch(step)
        x = torch.cat([xs[s][p:p + n] for s, n, p in step]).float().to(dev)
        d = torch.cat([ds[s][p:p + n] for s, n, p in step]).to(dtype).to(dev)
        x1, y = input_norm(x, d, [g.float().to(dev) for g in gains], [c.float().to(dev) for c in convs], eps, taps, b,
                           state, 8, dtype)
        close(x1, x.double().cpu() + d.double().cpu(), torch.float32)
        for i, (s, n, _) in enumerate(step):
            q0 = b.seq_meta_host[i][0]
            for o in range(k):
                ys[s][o].append(y[o][q0:q0 + n].double().cpu())
    for s in range(len(lengths)):
        for o in range(k):
            want = oracle.input_conv(oracle.rms(xs[s] + ds[s], eps) * gains[o], convs[o].t())
            close(torch.cat(ys[s][o]), want, dtype, bf16=1e-2)


def test_input_norm_embedding_rows_and_output_norm(run):
    dev, dtype = run
    W, taps = 48, 3
    emb = rnd(11, W, seed=1).to(dtype)
    pages = Pages(2, 2, 64, 8, [1, 0], dev, dtype)
    state = torch.zeros(2, 2 * W, device=dev)
    b = pages.batch([(0, 5, 0), (1, 2, 0)])
    ids = torch.tensor([3, 0, 10, 3, 7, 1, 1])
    b.input_ids = ids.to(dev)
    conv = rnd(taps, W, seed=2)
    g = torch.tensor([1.5])
    x, (y, ) = input_norm(None, None, [g.to(dev)], [conv.float().to(dev)], 1e-5, taps, b, state, 0, dtype,
                          embed=emb.to(dev))
    assert torch.equal(x.cpu(), emb[ids].float())
    e = emb[ids].double()
    want = torch.cat([oracle.input_conv(oracle.rms(p, 1e-5) * 1.5, conv.t()) for p in (e[:5], e[5:])])
    close(y, want, dtype, bf16=1e-2)
    idx = torch.tensor([6, 2], dtype=torch.int32, device=dev)
    d = rnd(7, W, seed=4).to(dtype).to(dev)
    got = norm_rows(x, d, idx, g.to(dev), 1e-5)
    close(got, oracle.rms(e[[6, 2]] + d.double().cpu()[[6, 2]], 1e-5) * 1.5, dtype, bf16=1e-2)


@pytest.mark.parametrize("W", [32, 37])
@pytest.mark.parametrize("sizes", [[1000], [1], [2], [70, 1, 33, 2, 32, 65]])
def test_gated_scan(run, W, sizes):
    dev, dtype = run
    lengths, slots = [1100 if sizes == [1000] else 260, 2, 64, 97], [2, 3, 0, 1]
    pages = Pages(4, 4, 64, 8, slots, dev, dtype)
    state = torch.full((4, 4 + W + (-W) % 4), 9.0, device=dev)
    bz, bx = rnd(W, seed=1) - 2.5, rnd(W, seed=2)  # slow gates: old tokens stay visible
    ps = [rnd(n, 3 * W, seed=30 + s, scale=1.5).to(dtype).double() for s, n in enumerate(lengths)]
    outs, last = [[] for _ in lengths], [None] * 4
    for step in portions(lengths, sizes):
        b = pages.batch(step)
        p = torch.cat([ps[s][q:q + n] for s, n, q in step]).to(dtype).to(dev)
        wide = torch.zeros(p.shape[0], W + 8, dtype=dtype, device=dev)
        gated_scan(p, bz.float().to(dev), bx.float().to(dev), wide[:, :W], b, state, 4)
        assert (wide[:, W:] == 0).all()
        for i, (s, n, _) in enumerate(step):
            q0 = b.seq_meta_host[i][0]
            outs[s].append(wide[q0:q0 + n, :W].double().cpu())
            last[s] = state[slots[s], 4:4 + W].double().cpu()
    eye = torch.eye(W, dtype=torch.float64)
    zero = torch.zeros_like(eye)
    w = {"z": torch.cat([eye, zero, zero], 1), "x": torch.cat([zero, eye, zero], 1),
         "g": torch.cat([zero, zero, eye], 1), "z.b": bz, "x.b": bx, "o": eye}
    for s in range(4):
        want, states = oracle.mingru(ps[s], w)
        close(torch.cat(outs[s]), want, dtype, bf16=1e-2)
        close(last[s][None], states[-1:], torch.float32)


@GPU
@pytest.mark.parametrize("M,N,K", [(1, 40, 24), (3, 37, 1048), (8, 64, 512)])
def test_fused_recurrence_step(M, N, K):
    dev = torch.device("cuda")
    slots = [(5 * i + 2) % 9 for i in range(M)]
    pages = Pages(M, M, 64, 8, slots, dev, torch.bfloat16)
    x = rnd(M, K, seed=1).to(torch.bfloat16).to(dev)
    w = rnd(3 * N, K, seed=2, scale=K**-0.5).to(torch.bfloat16).to(dev)
    bz, bx = rnd(N, seed=3).float().to(dev), rnd(N, seed=4).float().to(dev)
    seen = [0 if i == 1 else 4 + i for i in range(M)]
    b = pages.batch([(i, 1, seen[i]) for i in range(M)])
    s0 = rnd(9, 12 + N + (-N) % 4, seed=5).float().to(dev)
    s1, s2 = s0.clone(), s0.clone()
    out1 = torch.zeros(M, N + 3, dtype=torch.bfloat16, device=dev)
    out2 = torch.zeros_like(out1)
    recur_step(x, w, bz, bx, out1[:, :N], b, s1, 12)
    gated_scan(torch.nn.functional.linear(x, w), bz, bx, out2[:, :N], b, s2, 12)
    close(out1, out2, torch.bfloat16, bf16=1e-2)
    close(s1, s2, torch.bfloat16, bf16=5e-3)
    assert torch.equal(s1[:, :12], s0[:, :12])


@pytest.mark.parametrize("act", ["relu", "silu", "gelu_tanh"])
@pytest.mark.parametrize("T,I", [(5, 24), (1, 40), (3, 7)])
def test_gated_mlp_rows(run, act, T, I):
    dev, dtype = run
    gu = rnd(T, 2 * I, seed=1).to(dtype)
    wide = torch.zeros(T, I + 16, dtype=dtype, device=dev)
    glu_rows(gu.to(dev), act, wide[:, 16:])
    g, u = gu.double().split(I, 1)
    f = {"relu": torch.relu, "silu": torch.nn.functional.silu,
         "gelu_tanh": lambda z: 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z**3)))}[act]
    close(wide[:, 16:], f(g) * u, dtype, bf16=1e-2)
    assert (wide[:, :16] == 0).all()
    if dtype == torch.bfloat16:
        K = 264
        x, w = rnd(T, K, seed=2).to(dtype), rnd(2 * I, K, seed=3, scale=K**-0.5).to(dtype)
        wide.zero_()
        assert glu_gemv(x.to(dev), w.to(dev), act, wide[:, 16:])
        g, u = (x.double() @ w.double().t()).split(I, 1)
        close(wide[:, 16:], f(g) * u, dtype, bf16=1.5e-2)
        assert (wide[:, :16] == 0).all()


# (heads, dim, rot, rotated dims, rank, vdim, window): sizes of the plain and of the matrix-core kernels
SHAPES = {"odd": (3, 5, 6, 4, 7, 9, 11), "plain-prefill": (2, 8, 8, 8, 24, 24, 19), "mfma": (5, 24, 8, 8, 40, 16, 21),
          "mfma-rot-rest": (17, 40, 24, 12, 72, 48, 64), "no-window": (2, 32, 16, 16, 96, 80, 0),
          "wide": (2, 128, 64, 64, 264, 128, 130), "widest": (1, 192, 64, 64, 520, 208, 70),
          "window-1": (2, 16, 16, 16, 32, 32, 1), "18-heads": (18, 16, 16, 16, 200, 16, 40),
          "20-heads": (20, 16, 8, 8, 400, 16, 50), "full-64": (2, 48, 16, 16, 64, 64, 100),
          "full-128": (2, 64, 64, 64, 72, 128, 90)}


def _attention_case(name):
    H, dim, rot, rd, rank, vd, win = SHAPES[name]
    scale = min(0.3, 2.0 / math.sqrt(dim + rot))
    sh = LatentShape(heads=H, dim=dim, rot=rot, rot_dims=rd, rank=rank, vdim=vd, window=win, scale=scale, eps=1e-4)
    m = {"heads": H, "dim": dim, "rot_dim": rot, "vdim": vd, "kv_rank": rank, "scale": scale,
         "rot": {"dims": rd, "base": 700.0}, "mask": {"size": win or 10**9}}
    return sh, m


def _run_attention(sh, m, qds, w, sizes, dev, dtype, absorb_max=None, block_size=16, lengths=None, slots=None):
    """The op over portions of several sequences; returns every sequence's outputs."""
    lengths = lengths or [q.shape[0] for q in qds]
    slots = slots or list(range(len(qds)))[::-1]
    blocks = len(qds) * (-(-max(lengths) // block_size) + 1)
    pages = Pages(len(qds), blocks, block_size, sh.row, slots, dev, dtype)
    cos, sin = rope_tables(max(lengths) + 8, sh.rot_dims, m["rot"]["base"], device=dev)
    ukv = torch.cat([w["uk"], w["uv"]]).to(dtype).to(dev)
    uk = ukv[:sh.heads * sh.dim].view(sh.heads, sh.dim, sh.rank)
    uv = ukv[sh.heads * sh.dim:].view(sh.heads, sh.vdim, sh.rank)
    outs = [[] for _ in qds]
    for step in portions(lengths, sizes):
        b = pages.batch(step)
        qd = torch.cat([qds[s][p:p + n] for s, n, p in step]).to(dtype).to(dev)
        out = torch.zeros(qd.shape[0], sh.heads * sh.vdim + 8, dtype=dtype, device=dev)
        expand = dev.type == "cuda" and can_expand(sh, dtype)
        plan = make_plan(b.seq_meta_host, b.current_tokens, sh.window, expand, dev, absorb_max)
        latent_attention(qd[:, :sh.q_width], qd[:, sh.q_width:], sh, w["dkv.norm"].float().to(dev), uk, uv, ukv, cos, sin,
                         pages.cache, b, plan, out[:, :sh.heads * sh.vdim])
        assert (out[:, sh.heads * sh.vdim:] == 0).all()
        for i, (s, n, _) in enumerate(step):
            q0 = b.seq_meta_host[i][0]
            outs[s].append(out[q0:q0 + n, :sh.heads * sh.vdim].double().cpu())
    return [torch.cat(o) for o in outs]


def _oracle_attention(sh, m, qd, w):
    n = sh.q_width + sh.row
    eye = torch.eye(n, dtype=torch.float64)
    p = {"q": eye[:sh.q_width], "dkv": eye[sh.q_width:], "dkv.norm": w["dkv.norm"], "uk": w["uk"], "uv": w["uv"],
         "o": torch.eye(sh.heads * sh.vdim, dtype=torch.float64)}
    return oracle.latent_attention(qd, p, m, sh.eps)


def _attention_weights(sh, dtype):
    return {"uk": rnd(sh.heads * sh.dim, sh.rank, seed=2, scale=sh.rank**-0.5).to(dtype).double(),
            "uv": rnd(sh.heads * sh.vdim, sh.rank, seed=3, scale=sh.rank**-0.5).to(dtype).double(),
            "dkv.norm": (1 + 0.3 * rnd(sh.rank, seed=4)).to(dtype).double()}


@pytest.mark.parametrize("name", list(SHAPES))
@pytest.mark.parametrize("sizes", [[1000], [1], [2], [37, 1, 5, 2, 64, 90]])
def test_latent_attention(run, name, sizes):
    dev, dtype = run
    sh, m = _attention_case(name)
    if sizes == [1] and sh.rank > 200 and dev.type == "cpu":
        pytest.skip("slow without adding anything on the CPU")
    w = _attention_weights(sh, dtype)
    qds = [rnd(n, sh.q_width + sh.row, seed=40 + n).to(dtype).double() for n in (75, 2, 49)]
    got = _run_attention(sh, m, qds, w, sizes, dev, dtype)
    for g, qd in zip(got, qds):
        close(g, _oracle_attention(sh, m, qd, w), dtype, bf16=2e-2)


@pytest.mark.parametrize("name", ["mfma", "no-window", "wide", "full-64", "full-128"])
@pytest.mark.parametrize("sizes", [[1000], [190]])
def test_latent_attention_long_prompts(run, name, sizes):
    """Portions of several row blocks, with earlier keys before them."""
    dev, dtype = run
    if dev.type == "cpu":
        pytest.skip("the CPU implementation has one form")
    sh, m = _attention_case(name)
    w = _attention_weights(sh, dtype)
    qds = [rnd(n, sh.q_width + sh.row, seed=60 + n).to(dtype).double() for n in (330, 141)]
    got = _run_attention(sh, m, qds, w, sizes, dev, dtype, block_size=64)
    for g, qd in zip(got, qds):
        close(g, _oracle_attention(sh, m, qd, w), dtype, bf16=2e-2)


@pytest.mark.parametrize("name", ["odd", "mfma", "window-1", "no-window"])
@pytest.mark.parametrize("mode", ["prompt", "decode", "expanded-decode"])
def test_one_loud_key_at_every_distance(run, name, mode):
    """One key's score towers over all others; queries at every distance from it see exactly it, or do not."""
    dev, dtype = run
    sh, m = _attention_case(name)
    if mode == "expanded-decode" and not (dev.type == "cuda" and can_expand(sh, dtype)):
        pytest.skip("no expanded form here")
    n, bs = 70, 8
    w = _attention_weights(sh, dtype)
    # every head's query maps to the same latent direction: W_uk[h] has one row that reads latent 0
    uk = torch.zeros(sh.heads, sh.dim, sh.rank, dtype=torch.float64)
    uk[:, 0, 0] = 1.0
    w["uk"] = uk.view(-1, sh.rank)
    w["dkv.norm"] = torch.ones(sh.rank, dtype=torch.float64)
    for loud in (0, 7, 8, 15, 31, 33):
        qd = torch.zeros(n, sh.q_width + sh.row, dtype=torch.float64)
        q = qd[:, :sh.q_width].view(n, sh.heads, sh.dim + sh.rot)
        q[:, :, 0] = 64.0
        lat = qd[:, sh.q_width:sh.q_width + sh.rank]
        lat[:, 1:] = rnd(n, sh.rank - 1, seed=loud)
        lat[loud] = 0
        lat[loud, 0] = 1.0
        qd = qd.to(dtype).double()
        sizes = {"prompt": [n], "decode": [1], "expanded-decode": [2]}[mode]
        (got, ) = _run_attention(sh, m, [qd], w, sizes, dev, dtype, block_size=bs,
                                 absorb_max=1 if mode == "expanded-decode" else None)
        close(got, _oracle_attention(sh, m, qd, w), dtype, bf16=2e-2)
        value = w["uv"][:, 0] * math.sqrt(sh.rank)
        win = sh.window or 10**9
        for i in range(n):
            seen = 0 <= i - loud < win
            same = float((got[i] - value).norm() / value.norm())
            assert (same < 0.05) == seen, (loud, i, same)


# -----------------------------------------------------------------------------------------------
# models
# -----------------------------------------------------------------------------------------------
def _gru(width, ff=48):
    return {"type": "mingru", "mixer": {"width": width}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def _att(heads, dim, rot, rank, vdim, window, ff=48, base=900.0):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "kv_rank": rank, "vdim": vdim, "scale": 0.4,
                      "rot": {"dims": rot, "base": base}, "mask": {"size": window}},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


CONFIGS = {
    # two attention layers of different sizes, a looped recurrent layer, a layer without feed-forward
    "mixed": dict(vocab=131, width=64, canon={"taps": 4}, norm={"eps": 1e-5}, loop={"start": 1, "stop": 3, "times": 2},
                  layers=[_att(2, 24, 8, 40, 32, 9), _gru(48, 56), _att(3, 16, 16, 24, 16, 33, base=77.0),
                          _gru(40, None)]),
    "gru-only": dict(vocab=67, width=40, canon={"taps": 2}, norm={"eps": 1e-6}, loop=None,
                     layers=[_gru(56, 32), _gru(24, 24)]),
    "att-only": dict(vocab=90, width=48, canon={"taps": 1}, norm={"eps": 1e-4}, loop={"start": 0, "stop": 1, "times": 1},
                     layers=[_att(1, 8, 8, 16, 16, 1, None), _att(4, 40, 24, 48, 48, 100, 40)]),
    # sizes the matrix-core and vector paths do not take
    "odd": dict(vocab=61, width=37, canon={"taps": 3}, norm={"eps": 1e-6}, loop={"start": 0, "stop": 2, "times": 3},
                layers=[_gru(29, 31), _att(3, 5, 6, 7, 9, 12, 33)]),
}


def make_weights(cfg, seed=0):
    """Random weights, rounded to bfloat16 values; short memories (biased gates) would hide lost states, so the gates
    are slow, and queries and keys are loud enough that single keys matter."""
    g = torch.Generator().manual_seed(seed)
    w = {}

    def lin(name, rows, cols, scale=1.0):
        w[name] = torch.randn(rows, cols, generator=g) * scale * cols**-0.5

    W = cfg["width"]
    w["embed"] = torch.randn(cfg["vocab"], W, generator=g)
    for i, e in enumerate(cfg["layers"]):
        p, m = f"l{i}.", e["mixer"]
        if e["type"] == "mingru":
            n = m["width"]
            for k in ("z", "x", "g"):
                lin(f"{p}mix.{k}", n, W)
            w[p + "mix.z.b"] = torch.randn(n, generator=g) * 0.5 - 2.0
            w[p + "mix.x.b"] = torch.randn(n, generator=g)
            lin(p + "mix.o", W, n)
        else:
            H = m["heads"]
            lin(p + "mix.q", H * (m["dim"] + m["rot_dim"]), W, 2.0)
            lin(p + "mix.dkv", m["kv_rank"] + m["rot_dim"], W)
            w[p + "mix.dkv.norm"] = 1 + 0.3 * torch.randn(m["kv_rank"], generator=g)
            lin(p + "mix.uk", H * m["dim"], m["kv_rank"])
            lin(p + "mix.uv", H * m["vdim"], m["kv_rank"])
            lin(p + "mix.o", W, H * m["vdim"], 1.5)
        w[p + "norm1"] = torch.tensor(0.8 + 0.1 * i)
        w[p + "canon1"] = torch.randn(W, cfg["canon"]["taps"], generator=g) * 0.4
        if e["mlp"]:
            ff = e["mlp"]["ff"]
            w[p + "norm2"] = torch.tensor(1.3 - 0.1 * i)
            w[p + "canon2"] = torch.randn(W, cfg["canon"]["taps"], generator=g) * 0.4
            lin(p + "mlp.gate", ff, W)
            lin(p + "mlp.up", ff, W)
            lin(p + "mlp.down", W, ff)
    w["final.norm"] = torch.tensor(1.1)
    lin("head", cfg["vocab"], W)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


_CACHE = {}


def model(name):
    if name not in _CACHE:
        cfg = dict(CONFIGS[name], architecture="Gofasun")
        _CACHE[name] = (cfg, make_weights(cfg))
    return _CACHE[name]


def oracle_logits(name, tokens):
    key = (name, tuple(tokens))
    if key not in _CACHE:
        cfg, w = model(name)
        _CACHE[key] = oracle.forward(cfg, {k: v.double() for k, v in w.items()}, list(tokens))[0]
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
    for p, n in ((0, 20), (20, 1), (21, 1), (22, 11)):  # the other request goes on beside it
        lg, _ = eng.put([5], [torch.tensor(s[p:p + n])], capture_latents=False, logits_at=[range(n)])
        outs.append(lg.double().cpu())
    check_logits(torch.cat(outs), oracle_logits(name, s), run[1])
    check_logits(first[1], oracle_logits(name, tokens_of(name, 60, 21)), run[1])
    eng.flush(5)
    lg, _ = eng.put([9], [torch.tensor(s[:1])], capture_latents=False)  # one token in a slot full of old state
    check_logits(lg, oracle_logits(name, s)[:1], run[1])


def test_long_decoding(run):
    """Many single tokens, past every window, across pages; the batch's other sequence is at another position."""
    toks, other = tokens_of("mixed", 150, 30), tokens_of("mixed", 140, 31)
    steps = [[(0, 5, 0)], [(1, 2, 0)]] + [[(0, 1, 5 + i)] + ([(1, 1, 2 + i)] if i < 138 else []) for i in range(145)]
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
    with pytest.raises(ValueError):
        eng.put(["b"], [torch.tensor(b[:1])], capture_latents=False, logits_at=[[1]])


@pytest.mark.parametrize("name", ["mixed", "gru-only"])
def test_evict_and_restore(run, name):
    """HCache: cached rows come back from the returned latents, the recurrent state from the eviction."""
    eng = engine(name, run, blocks=8)
    s, o = tokens_of(name, 40, 3), tokens_of(name, 25, 4)
    lats = []
    for p, n in ((0, 22), (22, 1), (23, 1), (24, 9)):
        lg, (lat, ) = eng.put([1], [torch.tensor(s[p:p + n])])
        lats.append(lat.clone())
    eng.evict(1)
    feed(eng, [o], [[(0, 25, 0)]])  # other rows in the freed pages
    lat = torch.cat(lats, 1)
    with pytest.raises(RuntimeError):
        eng.restore_kv([1], [torch.tensor(s[:32])], [lat[:, :32]])
    eng.restore_kv([1], [torch.tensor(s[:33])], [lat])
    got = [eng.put([1], [torch.tensor(s[33 + i:34 + i])], capture_latents=False)[0].double().cpu() for i in range(7)]
    check_logits(torch.cat(got), oracle_logits(name, s)[33:], run[1])


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_greedy_generation(run, name):
    """The engine's own generation loop; compared with the plain implementation step by step along its own tokens."""
    prompt = tokens_of(name, 19, 5)
    eng = engine(name, run, blocks=8)
    out = eng.generate(1, torch.tensor(prompt), max_new_tokens=24)
    lg = oracle_logits(name, prompt + out)[len(prompt) - 1:-1]
    top = lg.max(-1).values
    picked = lg[torch.arange(24), out]
    assert ((top - picked) <= (1e-4 if run[1] == torch.float32 else 0.15)).all()
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
    them: states advance exactly once a step, and captured latents are the cached rows."""
    dev = torch.device("cuda")
    run = (dev, torch.bfloat16)
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
        want = oracle_logits("mixed", s)[11 + i % 3:17 + i % 3]
        check_logits(outs[True][:, i], want, torch.bfloat16)


def test_serialize_and_reload(run, tmp_path):
    eng = engine("mixed", run)
    s = tokens_of("mixed", 20, 6)
    a, = feed(eng, [s], [[(0, 20, 0)]])
    eng.serialize(str(tmp_path))
    conf = {"dtype": "fp32" if run[1] == torch.float32 else "bf16",
            "state_manager": {"max_context": 64, "kv_block_size": 16, "max_tracked_sequences": 2}}
    eng2 = build_engine_from_ds_checkpoint(str(tmp_path), conf, device=run[0], num_kv_blocks=4)
    b, = feed(eng2, [s], [[(0, 20, 0)]])
    assert torch.equal(a, b)


def test_weight_only_quantization():
    eng = engine("mixed", (torch.device("cpu"), torch.float32), quantization={"quantization_mode": "int8"})
    s = tokens_of("mixed", 20, 6)
    got, = feed(eng, [s], [[(0, 13, 0)], [(0, 7, 13)]])
    close(got, oracle_logits("mixed", s), torch.float32, f32=0.1)


def _tp_worker(rank, world, path):
    import hcache_deepspeed_amd as hds
    hds.init_distributed(dist_backend="gloo", verbose=False)
    cfg = dict(CONFIGS["mixed"], architecture="Gofasun")
    cfg["layers"] = [_att(2, 24, 8, 40, 32, 9), _gru(48, 56), _att(4, 16, 16, 24, 16, 33), _gru(40, None)]
    w = make_weights(cfg)
    spec = spec_from_hf(cfg)
    ec = RaggedInferenceEngineConfig.from_dict(dict(
        dtype="fp32", tensor_parallel={"tp_size": world},
        state_manager=dict(max_context=64, kv_block_size=16, max_tracked_sequences=2)))
    eng = InferenceEngineV2(spec, convert_hf(w, spec), ec, device=torch.device("cpu"), num_kv_blocks=4)
    s = tokens_of("mixed", 24, 8)
    got, = feed(eng, [s], [[(0, 17, 0)], [(0, 1, 17)], [(0, 6, 18)]])
    want = oracle.forward(cfg, {k: v.double() for k, v in w.items()}, s)[0]
    check_logits(got, want, torch.float32)


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
    assert eng.free_blocks == 3
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
    """A library of HybridTransformer.KERNEL_SOURCES alone exports every entry point the class's ops call."""
    import os
    import re

    from hcache_deepspeed_amd.inference.v2.hybrid import HybridTransformer
    from hcache_deepspeed_amd.ops import build, gated_scan, gemv, input_norm, latent_attention
    have = ""
    for f in HybridTransformer.KERNEL_SOURCES:
        with open(os.path.join(build.CSRC, "kernels", f)) as fh:
            have += fh.read()
    used = {"hds_glu_rows"}
    for mod in (gated_scan, gemv, input_norm, latent_attention):
        with open(mod.__file__) as fh:
            used |= set(re.findall(r"\)?\.(hds_\w+)\(", fh.read()))
    assert len(used) > 12
    for name in used:
        assert re.search(rf"HDS_EXPORT int {name}\(", have), name


def test_checkpoint_folder_and_registry(tmp_path):
    from safetensors.torch import save_file
    cfg, w = model("gru-only")
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    eng = build_hf_engine(str(tmp_path), {"dtype": "fp32", "state_manager": {"max_context": 64}},
                          device=torch.device("cpu"), num_kv_blocks=4)
    s = tokens_of("gru-only", 9, 1)
    lg, _ = eng.put([1], [torch.tensor(s)])
    check_logits(lg, oracle_logits("gru-only", s)[-1:], torch.float32)
    with pytest.raises(NotImplementedError):
        spec_from_hf({"architecture": "unknown"})
    with pytest.raises(NotImplementedError):
        spec_from_hf(dict(cfg, layers=[dict(cfg["layers"][0], type="other")]))
