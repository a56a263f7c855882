"""Fifotar on the ragged serving engine against the plain implementation in fifotar_oracle.py: every mechanism alone, then
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
from hcache_deepspeed_amd.inference.v2.arch import convert_hf, spec_from_hf
from hcache_deepspeed_amd.inference.v2.engine import (InferenceEngineV2, RaggedInferenceEngineConfig, SchedulingError,
                                                      transformer_class)
from hcache_deepspeed_amd.inference.v2.modules import (DSGatedMLPConfig, DSLinearConfig, DSMixerConfig,
                                                       instantiate_gated_mlp, instantiate_linear, instantiate_mixer)
from hcache_deepspeed_amd.ops import delta_rule as delta_op
from hcache_deepspeed_amd.ops.delta_rule import DeltaShape, delta_rule, make_delta_plan, step_ok
from hcache_deepspeed_amd.ops.latent_attention import LatentShape, can_expand, latent_attention, make_plan
from hcache_deepspeed_amd.ops.output_norm import rms_rows, sandwich_norm, softcap_
from hcache_deepspeed_amd.ops.paged import HeadShape, head_attention, head_blocks_ok, make_head_plan
from hcache_deepspeed_amd.ops.rope import rope_amplitude, rope_inv_freq, rope_tables

from . import fifotar_oracle as oracle
from .serving_utils import GPU, Pages, close, feed, portions, rnd, run, tokens  # noqa: F401

# -----------------------------------------------------------------------------------------------
# gated delta rule
# -----------------------------------------------------------------------------------------------
# (heads, kv heads, dim, vdim, taps): sizes of the vector and matrix-core kernels and of the plain ones
DELTAS = {"odd": (3, 1, 5, 7, 3), "odd-taps": (4, 2, 12, 20, 9), "one": (1, 1, 8, 8, 1), "small": (4, 2, 32, 64, 4),
          "wide-value": (2, 2, 24, 136, 2), "square-128": (2, 1, 128, 128, 4), "key-72": (6, 2, 72, 40, 5),
          "plain-key": (2, 1, 160, 48, 4), "value-256": (1, 1, 64, 256, 8)}


def _delta(name):
    H, G, d, e, taps = DELTAS[name]
    return DeltaShape(H, G, d, e, taps, 1e-4), {"heads": H, "kv_heads": G, "dim": d, "vdim": e, "conv": taps}


def _delta_weights(sh, seed=0, slow=True):
    """Convolutions, norm and decays; ``slow``: decays near one, so that early tokens still count at the end."""
    w = {"conv": rnd(sh.channels, sh.taps, seed=seed, scale=0.6), "norm": 1 + 0.3 * rnd(sh.vdim, seed=seed + 1),
         "A_log": rnd(sh.heads, seed=seed + 2, scale=0.5) - (5.0 if slow else 0.0), "dt_bias": rnd(sh.heads, seed=seed + 3)}
    return {k: v.float().double() for k, v in w.items()}


def _delta_oracle(sh, m, proj, w):
    """The oracle on projected rows: its projections pick them out."""
    G, H, d, e = sh.kv_heads, sh.heads, sh.dim, sh.vdim
    parts = torch.eye(sh.width, dtype=torch.float64).split([G * d, G * d, H * e, H * e, H, H])
    p = dict(zip(("q", "k", "v", "g", "b", "a"), parts), o=torch.eye(H * e).double())
    for k, c in zip(("q", "k", "v"), w["conv"].split([G * d, G * d, H * e])):
        p[k + ".conv"] = c
    return oracle.delta(proj, dict(p, A_log=w["A_log"], dt_bias=w["dt_bias"], norm=w["norm"]), m, sh.eps)


def _run_delta(sh, projs, w, sizes, dev, dtype, serial_max=None, monkeypatch=None, offset=8, slots=None):
    """The op over portions of several sequences, on states full of old values; returns every sequence's outputs."""
    if serial_max is not None:
        monkeypatch.setattr(delta_op, "SERIAL_MAX", serial_max)
    n = len(projs)
    pages = Pages(n, n, 16, 8, slots or list(range(n))[::-1], dev, dtype)
    state = torch.full((n + 1, offset + -(-sh.state_floats // 4) * 4 + 4), 3.0, device=dev)
    f = {k: v.float().to(dev) for k, v in w.items()}
    conv = f["conv"].t().contiguous()
    ld = -(-sh.width // 8) * 8
    single = dev.type == "cuda" and step_ok(sh)
    outs = [[] for _ in projs]
    for step in portions([p.shape[0] for p in projs], sizes):
        b = pages.batch(step)
        x = torch.full((b.current_tokens, ld), float("nan"), dtype=dtype, device=dev)
        x[:, :sh.width] = torch.cat([projs[s][p:p + k] for s, k, p in step]).to(dtype).to(dev)
        out = torch.zeros(b.current_tokens, sh.heads * sh.vdim + 8, dtype=dtype, device=dev)
        plan = make_delta_plan(b.seq_meta_host, b.current_sequences, b.max_new, single, dev)
        delta_rule(x, sh, conv, f["A_log"], f["dt_bias"], f["norm"], state, offset, b, plan, out[:, :sh.heads * sh.vdim])
        assert (out[:, sh.heads * sh.vdim:] == 0).all() and (state[n] == 3.0).all()
        assert (state[:, :offset] == 3.0).all() and (state[:, -4:] == 3.0).all()
        for i, (s, k, _) in enumerate(step):
            q0 = b.seq_meta_host[i][0]
            outs[s].append(out[q0:q0 + k, :sh.heads * sh.vdim].double().cpu())
    return [torch.cat(o) for o in outs]


@pytest.mark.parametrize("name", list(DELTAS))
@pytest.mark.parametrize("sizes", [[1000], [1], [2], [37, 1, 5, 2, 64, 90]])
def test_delta(run, name, sizes):
    dev, dtype = run
    sh, m = _delta(name)
    w = _delta_weights(sh)
    projs = [rnd(n, sh.width, seed=40 + n).to(dtype).double() for n in (75, 2, 41)]
    got = _run_delta(sh, projs, w, sizes, dev, dtype)
    for g, x in zip(got, projs):
        close(g, _delta_oracle(sh, m, x, w), dtype, f32=5e-5, bf16=3e-2)


@pytest.mark.parametrize("name", ["small", "square-128", "key-72", "wide-value"])
@pytest.mark.parametrize("sizes", [[1000], [63, 64, 65], [130, 1, 17]])
@pytest.mark.parametrize("slow", [True, False])
def test_delta_long_portions(run, name, sizes, slow):
    """Several chunks of the matrix-core scan, ends inside and at the edges of chunks, decays near one and near zero."""
    dev, dtype = run
    if dev.type == "cpu":
        pytest.skip("the CPU implementation has one form")
    sh, m = _delta(name)
    w = _delta_weights(sh, slow=slow)
    projs = [rnd(n, sh.width, seed=60 + n).to(dtype).double() for n in (200, 128, 129)]
    got = _run_delta(sh, projs, w, sizes, dev, dtype)
    for g, x in zip(got, projs):
        close(g, _delta_oracle(sh, m, x, w), dtype, f32=5e-5, bf16=3e-2)


@GPU
@pytest.mark.parametrize("name", ["small", "square-128", "key-72", "value-256"])
def test_chunk_scan_is_the_serial_scan(name, monkeypatch):
    """Both forms keep 32-bit states: from the same bfloat16 rows they differ by 32-bit rounding, before the outputs are
    rounded (nearly all outputs are the same bfloat16 number)."""
    dev, dtype = torch.device("cuda"), torch.bfloat16
    print(f"chunk / serial {name}", flush=True)
    sh, _ = _delta(name)
    w = _delta_weights(sh, seed=9)
    projs = [rnd(n, sh.width, seed=80 + n).to(dtype).double() for n in (150, 77)]
    a = _run_delta(sh, projs, w, [1000], dev, dtype, serial_max=0, monkeypatch=monkeypatch)
    b = _run_delta(sh, projs, w, [1000], dev, dtype, serial_max=10**6, monkeypatch=monkeypatch)
    for x, y in zip(a, b):
        assert ((x - y).abs() <= 0.008 * x.abs() + 2e-5 * x.abs().mean()).all()  # one step of bfloat16
        assert (x != y).double().mean() < 0.01


def test_delta_mechanisms_show(run):
    """Single pieces of the rule where a slip would hide in random data: a written value is read back by its key at any
    distance, replaced by a second write, halved by a decay of one half; the read-out sees its own token's write."""
    dev, dtype = run
    sh = DeltaShape(2, 1, 8, 8, 2, 1e-6)
    H, d, e = 2, 8, 8
    n = 40
    for sizes in ([1000], [1], [7, 1, 2]):
        x = torch.zeros(n, sh.width, dtype=torch.float64)
        q, k, v, g, b, a = x.split([d, d, H * e, H * e, H, H], 1)
        w = {"conv": torch.zeros(sh.channels, 2).double(), "norm": torch.ones(e).double(),
             "A_log": torch.zeros(H).double(), "dt_bias": torch.zeros(H).double()}
        w["conv"][:, 1] = 1.0  # the current token alone
        g[:] = 8.0
        b[:] = -40.0           # writes nothing ...
        a[:] = -40.0           # keeps everything
        q[:, 0] = 20.0         # reads with key 0
        k[:, 1] = 20.0
        k[3], k[20] = 0, 0
        k[3, 0] = k[20, 0] = 20.0
        b[3] = b[20] = 40.0    # ... but at 3 and 20, where the key is key 0
        v[:] = rnd(n, H * e, seed=1)
        v[3], v[20] = rnd(H * e, seed=2).abs() + 1, rnd(H * e, seed=3).abs() + 1
        (got, ) = _run_delta(sh, [x.to(dtype).double()], w, sizes, dev, dtype)
        for lo, hi, src in ((3, 20, 3), (20, n, 20)):
            want = oracle.silu(v[src].to(dtype).double()).view(H, e)
            want = want / want.pow(2).mean(-1, keepdim=True).sqrt() * 8.0
            for i in range(lo, hi):
                assert (got[i].view(H, e) - want).abs().max() < 0.15, (sizes, i)
        assert got[:3].abs().max() < 1e-2
    # the state itself: unnormed read-outs of a decaying state, by the ratio to a second head column kept alive
    x = torch.zeros(4, sh.width, dtype=torch.float64)
    q, k, v, g, b, a = x.split([d, d, H * e, H * e, H, H], 1)
    q[:, :2] = 20.0
    k[0, 0] = k[1, 1] = k[2, 2] = k[3, 2] = 20.0
    b[:2], b[2:] = 40.0, -40.0
    v[0, 0] = v[1, 1] = 20.0   # value 0 at token 0 by key 0, value 1 at token 1 by key 1
    v[0, e] = v[1, e + 1] = 20.0
    g[:] = 8.0
    w["A_log"][:] = math.log(math.log(2) / math.log1p(1.0))
    a[:] = math.log(math.expm1(math.log(2)))  # softplus = log 2, times exp(A_log) = 1: every token halves the state
    w["A_log"][:] = 0.0
    (got, ) = _run_delta(sh, [x], w, [1000], dev, torch.float32 if dtype == torch.float32 else dtype)
    for i in (1, 2, 3):
        assert abs(float(got[i, 0] / got[i, 1]) - 0.5) < 0.02  # token 0's value decayed once more than token 1's


def test_delta_state_of_another_slot(run):
    """Sequences swap nothing: each keeps its own state and convolution inputs whatever slots and orders are used."""
    dev, dtype = run
    sh, m = _delta("small")
    w = _delta_weights(sh)
    projs = [rnd(n, sh.width, seed=n).to(dtype).double() for n in (9, 30, 17, 4)]
    for sizes in ([1], [3, 1], [2, 9]):
        got = _run_delta(sh, projs, w, sizes, dev, dtype, slots=[2, 0, 3, 1])
        for g, x in zip(got, projs):
            close(g, _delta_oracle(sh, m, x, w), dtype, f32=5e-5, bf16=3e-2)


# -----------------------------------------------------------------------------------------------
# attention
# -----------------------------------------------------------------------------------------------
# (heads, kv heads, dim, vdim, chunk)
HEADS = {"odd": (3, 1, 5, 7, 11), "exact-64": (4, 2, 64, 64, 33), "exact-128": (8, 1, 128, 128, 40),
         "uneven": (6, 3, 24, 56, 70), "12-per-key": (12, 1, 32, 32, 64), "chunk-1": (3, 3, 16, 16, 1),
         "wide-value": (2, 1, 16, 200, 18), "no-chunk": (2, 2, 80, 80, 0), "plain-wide": (2, 2, 264, 24, 25)}


def _heads(name, softcap=9.0):
    H, G, d, e, chunk = HEADS[name]
    sh = HeadShape(heads=H, kv_heads=G, dim=d, vdim=e, window=0, scale=2.5 / math.sqrt(d), eps=1e-5, gated=True,
                   gate_width=e, chunk=chunk, softcap=softcap)
    return sh, {"heads": H, "kv_heads": G, "dim": d, "vdim": e, "scale": sh.scale, "softcap": softcap,
                "mask": {"size": chunk} if chunk else None}


def _run_heads(sh, qkvs, sizes, dev, dtype, decode_max=None, block_size=16, values=None, mix=0.3):
    lengths = [q.shape[0] for q in qkvs]
    blocks = len(qkvs) * (-(-max(lengths) // block_size) + 1)
    pages = Pages(len(qkvs), blocks, block_size, sh.row, list(range(len(qkvs)))[::-1], dev, dtype)
    sink = torch.zeros(sh.heads, device=dev)
    lam = torch.tensor([mix], device=dev)
    outs = [[] for _ in qkvs]
    ld = -(-sh.width // 8) * 8
    for step in portions(lengths, sizes):
        b = pages.batch(step)
        qkv = torch.full((b.current_tokens, ld), float("nan"), dtype=dtype, device=dev)
        qkv[:, :sh.width] = torch.cat([qkvs[s][p:p + n] for s, n, p in step]).to(dtype).to(dev)
        out = torch.zeros(b.current_tokens, sh.heads * sh.vdim + 8, dtype=dtype, device=dev)
        blocks_on = dev.type == "cuda" and b.max_new > 1 and head_blocks_ok(sh, dtype)
        plan = make_head_plan(b.seq_meta_host, b.current_tokens, sh.heads, sh.kv_heads, blocks_on, dev, decode_max)
        first = None
        if values is not None:  # in a wider matrix, as the first layer's projection holds them
            wide = torch.zeros(b.current_tokens, 8 + values[0].shape[1] + 8 - values[0].shape[1] % 8, dtype=dtype, device=dev)
            first = wide[:, 8:8 + values[0].shape[1]]
            first.copy_(torch.cat([values[s][p:p + n] for s, n, p in step]).to(dtype))
        head_attention(qkv, sh, None, None, sink, pages.cache, b, plan, out[:, :sh.heads * sh.vdim], first, lam)
        assert (out[:, sh.heads * sh.vdim:] == 0).all()
        for i, (s, n, _) in enumerate(step):
            q0 = b.seq_meta_host[i][0]
            outs[s].append(out[q0:q0 + n, :sh.heads * sh.vdim].double().cpu())
    return [torch.cat(o) for o in outs]


def _oracle_heads(sh, m, qkv, first=None, mix=0.3):
    parts = torch.eye(sh.width, dtype=torch.float64).split(
        [sh.heads * sh.dim, sh.kv_heads * sh.dim, sh.kv_heads * sh.vdim, sh.width - sh.qkv_width])
    p = dict(zip(("q", "k", "v", "g"), parts), o=torch.eye(sh.heads * sh.vdim).double(), vmix=mix)
    f = None if first is None else first.view(-1, sh.kv_heads, sh.vdim)
    return oracle.attention(qkv, p, m, f)[0]


@pytest.mark.parametrize("name", list(HEADS))
@pytest.mark.parametrize("sizes", [[1000], [1], [2], [37, 1, 5, 2, 64, 90]])
@pytest.mark.parametrize("mixed", [False, True])
def test_attention(run, name, sizes, mixed):
    dev, dtype = run
    sh, m = _heads(name)
    mix = float(torch.tensor(0.3))
    qkvs = [rnd(n, sh.width, seed=40 + n).to(dtype).double() for n in (75, 2, 41)]
    vals = [rnd(q.shape[0], sh.kv_heads * sh.vdim, seed=7).to(dtype).double() for q in qkvs] if mixed else None
    got = _run_heads(sh, qkvs, sizes, dev, dtype, values=vals, mix=mix)
    for i, (g, x) in enumerate(zip(got, qkvs)):
        close(g, _oracle_heads(sh, m, x, vals[i] if mixed else None, mix), dtype, f32=4e-5, bf16=2e-2)


def test_projection_in_two_products(run, monkeypatch):
    """Long steps run gates, or b and a, as a product of their own."""
    from hcache_deepspeed_amd.inference.v2.modules import implementations
    dev, dtype = run
    toks = tokens_of("mixed", 150, 4)
    calls = []
    monkeypatch.setattr(implementations, "SPLIT_ROWS", 20)
    monkeypatch.setattr(implementations, "_tile_rounds", lambda rows, cols: calls.append(cols) or len(calls))
    eng = engine("mixed", run, blocks=12)
    got, = feed(eng, [toks], [[(0, 100, 0)], [(0, 19, 100)], [(0, 31, 119)]])
    check_logits(got, oracle_logits("mixed", toks), dtype)
    assert len(calls) == 2 * 2 * 2


@pytest.mark.parametrize("name", ["exact-64", "exact-128", "uneven", "12-per-key"])
@pytest.mark.parametrize("sizes", [[1000], [90]])
def test_attention_long_prompts(run, name, sizes):
    """Portions of several row blocks, chunks that end in the middle of a block's rows and keys."""
    dev, dtype = run
    if dev.type == "cpu":
        pytest.skip("the CPU implementation has one form")
    sh, m = _heads(name)
    qkvs = [rnd(n, sh.width, seed=60 + n).to(dtype).double() for n in (210, 141)]
    got = _run_heads(sh, qkvs, sizes, dev, dtype, block_size=64)
    for g, x in zip(got, qkvs):
        close(g, _oracle_heads(sh, m, x), dtype, f32=4e-5, bf16=2e-2)


@pytest.mark.parametrize("name", ["odd", "exact-64", "uneven", "chunk-1", "no-chunk"])
@pytest.mark.parametrize("mode", ["prompt", "decode", "short-blocks"])
def test_one_loud_key_at_every_distance(run, name, mode):
    """One key's score towers over all others and the sink; queries of its chunk after it see exactly it, others do
    not."""
    dev, dtype = run
    sh, m = _heads(name, softcap=60.0)
    if mode == "short-blocks" and not (dev.type == "cuda" and head_blocks_ok(sh, dtype)):
        pytest.skip("no block form here")
    n, bs = 80, 8
    for loud in (0, 7, 8, 15, 32, 33, 69, 70):
        x = torch.zeros(n, sh.width, dtype=torch.float64)
        q, k, v, g = x.split([sh.heads * sh.dim, sh.kv_heads * sh.dim, sh.kv_heads * sh.vdim, sh.heads * sh.vdim], 1)
        q.view(n, sh.heads, sh.dim)[:, :, 0] = 8.0 / sh.scale
        v[:] = rnd(n, v.shape[1], seed=loud)
        g[:] = 30.0
        k.view(n, sh.kv_heads, sh.dim)[loud, :, 0] = 4.0
        x = x.to(dtype).double()
        sizes = {"prompt": [n], "decode": [1], "short-blocks": [2]}[mode]
        (got, ) = _run_heads(sh, [x], sizes, dev, dtype, block_size=bs, decode_max=0 if mode == "short-blocks" else None)
        value = v[loud].to(dtype).double().view(sh.kv_heads, sh.vdim).repeat_interleave(sh.heads // sh.kv_heads, 0)
        value = value.reshape(-1)
        chunk = sh.chunk or 10**9
        for i in range(n):
            same = float((got[i] - value).norm() / value.norm())
            assert (same < 0.05) == (i >= loud and i // chunk == loud // chunk), (loud, i, same)


@pytest.mark.parametrize("name", ["odd", "exact-64", "12-per-key"])
@pytest.mark.parametrize("sizes", [[1000], [1]])
def test_sink_cap_and_gates(run, name, sizes):
    """A lone key of score s weighs e^s / (1 + e^s); scores above the cap stay below it; every element has its own gate."""
    dev, dtype = run
    sh, m = _heads(name, softcap=2.0)
    n = 1
    x = torch.zeros(n, sh.width, dtype=torch.float64)
    q, k, v, g = x.split([sh.heads * sh.dim, sh.kv_heads * sh.dim, sh.kv_heads * sh.vdim, sh.heads * sh.vdim], 1)
    v[:], g[:] = 1.0, 40.0
    g[:, 1] = -40.0
    k.view(n, sh.kv_heads, sh.dim)[:, :, 0] = 1.0
    for s in (0.0, 0.5, -1.0, 100.0, -100.0):
        q.view(n, sh.heads, sh.dim)[:, :, 0] = s / sh.scale
        (got, ) = _run_heads(sh, [x.to(dtype).double()], sizes, dev, dtype)
        want = 1 / (1 + math.exp(-2.0 * math.tanh(s / 2.0)))
        assert abs(float(got[0, 0]) - want) < (1e-5 if dtype == torch.float32 else 1e-2), (s, got[0, 0], want)
        assert abs(float(got[0, 1])) < 1e-9


def test_yarn_frequencies():
    for n, base, sc in ((16, 500000.0, (8.0, 32.0, 1.0, 512)), (64, 10000.0, (40.0, 32.0, 1.0, 4096)),
                        (6, 1000.0, (2.0, 8.0, 2.0, 100)), (2, 50.0, (4.0, 3.0, 3.0, 64)), (10, 10000.0, None)):
        rot = {"dims": n, "base": base}
        ours = None
        if sc:
            rot["scaling"] = {"factor": sc[0], "fast": sc[1], "slow": sc[2], "original": sc[3]}
            ours = {"rope_type": "yarn", "factor": sc[0], "beta_fast": sc[1], "beta_slow": sc[2],
                    "original_max_position_embeddings": sc[3]}
        want, amp = oracle.frequencies(rot)
        assert torch.allclose(rope_inv_freq(n, base, ours), torch.tensor(want, dtype=torch.float64), rtol=1e-12)
        assert abs(rope_amplitude(ours) - amp) < 1e-12
        cos, sin = rope_tables(3000, n, base, ours)
        a = 2999 * torch.tensor(want, dtype=torch.float64)
        assert torch.allclose(cos[2999].double(), amp * a.cos(), atol=1e-6)
        assert torch.allclose(sin[2999].double(), amp * a.sin(), atol=1e-6)
        assert cos[0].allclose(torch.tensor(amp, dtype=torch.float32).expand_as(cos[0]))


# (heads, dim, rot dim, rotated, kv rank, q rank, vdim): vector and matrix-core sizes, plain ones, a partly rotated part
LATENTS = {"exact": (4, 32, 16, 16, 64, 48, 32), "odd": (3, 5, 6, 6, 11, 9, 7), "partly": (2, 24, 16, 8, 40, 32, 16),
           "half-dims": (2, 20, 12, 4, 24, 24, 20), "wide": (16, 128, 64, 64, 256, 96, 128)}


def _mixer(kind, params, W, dev, dtype, weights, eps=1e-4):
    """The registered mixer with its linears and its weights on the device."""
    mix = instantiate_mixer(DSMixerConfig(kind, W, params, eps, 1, dtype))
    if hasattr(mix, "bind_tables"):
        mix.bind_tables(*rope_tables(512, mix.shape.rot_dims, mix.rope_base, mix.rope_scaling, device=dev))
    lins = {k: instantiate_linear(DSLinearConfig(*io)) for k, io in {"in.w": (W, mix.in_width), **mix.extra_linears()}.items()}
    raw = mix.shard(weights, lambda t: t, lambda t: t)
    mats = ("in.w", "o.w", "uq.w", "ukv.w")
    w = {k: None if v is None else v.to(dtype if k in mats else torch.float32).contiguous().to(dev) for k, v in raw.items()}
    return mix, lins, w


@pytest.mark.parametrize("name", list(LATENTS))
@pytest.mark.parametrize("sizes", [[1000], [1], [2], [37, 1, 5, 2, 64, 90]])
def test_latent_attention(run, name, sizes):
    """The mixer from its input rows: query latent, half rotation with YaRN, gate per head."""
    dev, dtype = run
    H, d, r, rd, rank, qr, e = LATENTS[name]
    W, eps = 40, 1e-4
    sc = {"factor": 6.0, "fast": 20.0, "slow": 1.5, "original": 60}
    m = {"heads": H, "dim": d, "rot_dim": r, "kv_rank": rank, "q_rank": qr, "vdim": e, "scale": 1.4 * (d + r)**-0.5,
         "rot": {"base": 300.0, "dims": rd, "scaling": sc}}
    p = {"dq": rnd(qr, W, seed=1, scale=W**-0.5), "dq.norm": 1 + 0.2 * rnd(qr, seed=2),
         "uq": rnd(H * (d + r), qr, seed=3, scale=1.5 * qr**-0.5), "dkv": rnd(rank + r, W, seed=4, scale=W**-0.5),
         "dkv.norm": 1 + 0.2 * rnd(rank, seed=5), "uk": rnd(H * d, rank, seed=6, scale=1.5 * rank**-0.5),
         "uv": rnd(H * e, rank, seed=7, scale=rank**-0.5), "g": rnd(H, W, seed=8, scale=W**-0.5),
         "o": torch.eye(H * e).double()}
    p = {k: v.to(torch.bfloat16).double() for k, v in p.items()}
    params = spec_from_hf({"architecture": "Fifotar", "vocab": 4, "width": W, "norm": {"eps": eps}, "residual_mult": 1.0,
                           "embedding": {"scale": 1.0}, "logit_softcap": None,
                           "layers": [{"type": "latent_attention", "mixer": m, "mlp": None}]}).layers[0]["mixer"]
    mix, lins, w = _mixer("latent_attention", params, W, dev, dtype, p, eps)
    xs = [rnd(n, W, seed=20 + n).to(dtype).double() for n in (75, 2, 41)]
    pages = Pages(3, 18, 16, mix.cache_row, [2, 0, 1], dev, dtype)
    outs = [[] for _ in xs]
    for step in portions([x.shape[0] for x in xs], sizes):
        b = pages.batch(step)
        x = torch.cat([xs[s][q:q + n] for s, n, q in step]).to(dtype).to(dev)
        out = torch.zeros(b.current_tokens, mix.out_width, dtype=dtype, device=dev)
        mix(x, w, lins, out, b, pages.cache, None, 0)
        for i, (s, n, _) in enumerate(step):
            q0 = b.seq_meta_host[i][0]
            outs[s].append(out[q0:q0 + n].double().cpu())
    for o, x in zip(outs, xs):
        close(torch.cat(o), oracle.latent_attention(x, p, m, eps), dtype, f32=5e-5, bf16=4e-2)


@pytest.mark.parametrize("name", ["exact", "odd"])
@pytest.mark.parametrize("sizes", [[300], [1], [131, 2, 17]])
def test_latent_attention_finds_one_key_at_any_distance(run, name, sizes):
    """One latent's score towers over the others': every later query, next to it or hundreds of tokens on, gives back its
    value times the head's gate, earlier ones do not see it."""
    dev, dtype = run
    H, d, r, rd, rank, _, e = LATENTS[name]
    n = 300
    sh = LatentShape(heads=H, dim=d, rot=r, rot_dims=rd, rank=rank, vdim=e, window=0, scale=0.5, eps=1e-6, gated=True)
    cos, sin = rope_tables(512, rd, 1000.0, device=dev)
    uk = torch.zeros(H, d, rank, dtype=torch.float64)
    uk[:, 0, 0] = 1.0
    uv = rnd(H, e, rank, seed=1)
    ukv = torch.cat([uk.reshape(H * d, rank), uv.reshape(H * e, rank)]).to(dtype).to(dev)
    for loud in (0, 1, 63, 64, 130):
        q = torch.zeros(n, H, d + r, dtype=torch.float64)
        q[:, :, 0] = 60.0
        ckr = torch.zeros(n, rank + r, dtype=torch.float64)
        ckr[:, 1:rank] = rnd(n, rank - 1, seed=loud + 2)
        ckr[loud] = 0.0
        ckr[loud, 0] = 3.0
        gate = torch.full((n, H), 0.7, dtype=torch.float64)
        pages = Pages(1, 5, 64, sh.row, [0], dev, dtype)
        outs = []
        for step in portions([n], sizes):
            (_, k, p), = step
            b = pages.batch(step)
            t = lambda x: x[p:p + k].to(dtype).to(dev).contiguous()  # noqa: E731
            out = torch.zeros(k, H * e, dtype=dtype, device=dev)
            expand = dev.type == "cuda" and b.max_new > 1 and can_expand(sh, dtype)
            plan = make_plan(b.seq_meta_host, k, 0, expand, dev)
            latent_attention(t(q).view(k, -1), t(ckr), sh, torch.ones(rank, device=dev), ukv[:H * d].view(H, d, rank),
                             ukv[H * d:].view(H, e, rank), ukv, cos, sin, pages.cache, b, plan, out, t(gate))
            outs.append(out.double().cpu())
        got = torch.cat(outs)
        want = (uv[:, :, 0].to(dtype).double() * rank**0.5 * torch.sigmoid(torch.tensor(0.7))).reshape(-1)
        for i in range(n):
            same = float((got[i] - want).norm() / want.norm())
            assert (same < 0.05) == (i >= loud), (loud, i, same)


# -----------------------------------------------------------------------------------------------
# norms, feed-forward, logits
# -----------------------------------------------------------------------------------------------
@pytest.mark.parametrize("T,W", [(5, 64), (1, 37), (3, 2048), (100, 72), (2, 4104), (70, 1536), (1, 9000), (80, 4096),
                                 (65, 37), (3, 320), (1, 8192)])
def test_sandwich_norm(run, T, W):
    dev, dtype = run
    x, d = rnd(T, W, seed=1, scale=3.0).float().double(), rnd(T, W, seed=2, scale=0.1).to(dtype).double()
    g, gn = ((1 + 0.5 * rnd(W, seed=s)).float().double() for s in (3, 4))
    f = lambda t: t.float().to(dev)  # noqa: E731
    eps = 1e-3
    want = x + oracle.rms(d, eps, g)
    x1, y = sandwich_norm(f(x), d.to(dtype).to(dev), f(g), f(gn), eps, dtype)
    close(x1, want, torch.float32)
    close(y, oracle.rms(want, eps, gn), dtype, bf16=5e-3)
    idx = torch.tensor([T - 1, 0], dtype=torch.int32, device=dev)
    none, y = sandwich_norm(f(x), d.to(dtype).to(dev), f(g), f(gn), eps, dtype, idx=idx)
    assert none is None
    close(y, oracle.rms(want, eps, gn)[[T - 1, 0]], dtype, bf16=5e-3)
    emb = rnd(11, W, seed=1).to(dtype)
    ids = torch.randint(0, 11, (T, ), generator=torch.Generator().manual_seed(1))
    x1, y = sandwich_norm(None, None, None, f(gn), eps, dtype, embed=(emb.to(dev), ids.to(dev), 2.5))
    close(x1, emb.double()[ids] * 2.5, torch.float32, f32=1e-6)
    close(y, oracle.rms(emb.double()[ids] * 2.5, eps, gn), dtype, bf16=5e-3)


@pytest.mark.parametrize("T,W,ld", [(5, 64, 80), (9, 37, 50), (1, 2500, 2501), (300, 1024, 1200), (3, 4096, 4096)])
def test_row_norm(run, T, W, ld):
    dev, dtype = run
    x = rnd(T, ld, seed=1).to(dtype)
    g = (1 + 0.5 * rnd(W, seed=3)).float()
    close(rms_rows(x.to(dev)[:, :W], g.to(dev), 1e-3), oracle.rms(x.double()[:, :W], 1e-3, g.double()), dtype, bf16=5e-3)


def test_logit_cap(run):
    dev, dtype = run
    x = rnd(7, 333, seed=1, scale=40.0).to(dtype)
    close(softcap_(x.clone().to(dev), 30.0), oracle.softcap(x.double(), 30.0), dtype, f32=1e-6, bf16=5e-3)


@pytest.mark.parametrize("T", [1, 2, 40])
@pytest.mark.parametrize("W,ff,limit", [(64, 48, 1.5), (40, 37, 0.4), (128, 256, 50.0)])
def test_clamped_feed_forward(run, T, W, ff, limit):
    dev, dtype = run
    p = {k: rnd(ff, W, seed=s, scale=2 * W**-0.5).to(dtype).double() for k, s in (("gate", 1), ("up", 2))}
    x = rnd(T, W, seed=3).to(dtype).double()
    mlp = instantiate_gated_mlp(DSGatedMLPConfig(W, ff, "clamped", limit))
    lin = instantiate_linear(DSLinearConfig(W, 2 * ff))
    out = torch.zeros(T, ff, dtype=dtype, device=dev)
    mlp(x.to(dtype).to(dev), torch.cat([p["gate"], p["up"]]).to(dtype).to(dev), lin, out)
    want = oracle.feed_forward(x, dict(p, down=torch.eye(ff).double()), limit)
    close(out, want, dtype, bf16=2e-2)


# -----------------------------------------------------------------------------------------------
# models
# -----------------------------------------------------------------------------------------------
def _mlp(ff, limit=1.5):
    return {"kind": "dense", "ff": ff, "limit": limit}


def _del(H, G, d, e, taps, mlp=None):
    return {"type": "delta", "mixer": {"heads": H, "kv_heads": G, "dim": d, "vdim": e, "conv": taps}, "mlp": mlp}


def _lat(H, d, r, rank, qr, e, mlp=None, base=1000.0, sc=(4.0, 16.0, 1.0, 48)):
    scaling = dict(zip(("factor", "fast", "slow", "original"), sc)) if sc else None
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": H, "dim": d, "rot_dim": r, "kv_rank": rank, "q_rank": qr, "vdim": e,
                      "scale": 1.7 * (d + r)**-0.5, "rot": {"base": base, "dims": r, "scaling": scaling}}}


def _att(H, G, d, e, chunk, mlp=None, mix=True, cap=12.0):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": H, "kv_heads": G, "dim": d, "vdim": e, "scale": 1.5 * d**-0.5, "softcap": cap,
                      "mask": {"size": chunk}, "v_mix": mix}}


CONFIGS = {
    # an unmixed attention layer before, between and after the mixed ones, feed-forwards in some layers
    "mixed": dict(vocab=131, width=64, norm={"eps": 1e-5}, embedding={"scale": 7.0}, residual_mult=0.7,
                  logit_softcap=25.0,
                  layers=[_att(4, 4, 24, 16, 13, _mlp(40), mix=False), _del(4, 2, 16, 24, 3, _mlp(72, 0.8)),
                          _att(4, 2, 16, 24, 20), _lat(4, 24, 8, 40, 32, 16, _mlp(48)), _del(2, 2, 32, 16, 4),
                          _att(6, 2, 32, 24, 33, _mlp(56)), _att(2, 1, 16, 32, 7, mix=False),
                          _att(8, 2, 8, 24, 50, cap=40.0)]),
    # begins with a recurrence, one value of everything
    "first-delta": dict(vocab=90, width=40, norm={"eps": 1e-3}, embedding={"scale": 1.0}, residual_mult=1.0,
                        logit_softcap=8.0,
                        layers=[_del(1, 1, 8, 8, 1, _mlp(8, 3.0)), _att(1, 1, 8, 8, 16, mix=False),
                                _lat(1, 8, 8, 8, 8, 8, sc=None)]),
    "wide": dict(vocab=67, width=128, norm={"eps": 1e-6}, embedding={"scale": 5.0}, residual_mult=0.4,
                 logit_softcap=30.0, layers=[_lat(16, 64, 32, 128, 96, 64, _mlp(136)), _del(2, 1, 128, 128, 4),
                                             _att(8, 1, 128, 128, 64, _mlp(256))]),
    # nothing that can be left out
    "bare": dict(vocab=75, width=48, norm={"eps": 1e-5}, embedding={"scale": 3.0}, residual_mult=0.6, logit_softcap=None,
                 layers=[dict(_att(4, 2, 16, 16, 8), mixer={"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 16, "scale": 0.3}),
                         _lat(4, 16, 8, 24, 32, 24, sc=None), _del(3, 3, 16, 8, 2)]),
    # sizes the matrix-core and vector paths do not take
    "odd": dict(vocab=61, width=37, norm={"eps": 1e-6}, embedding={"scale": 5.0}, residual_mult=0.9, logit_softcap=11.0,
                layers=[_del(3, 1, 5, 7, 3, _mlp(11)), _att(3, 1, 5, 7, 12), _lat(3, 5, 6, 9, 7, 7, _mlp(13)),
                        _att(2, 1, 9, 7, 5), _del(2, 2, 3, 10, 2)]),
}


def make_weights(cfg, seed=0):
    """Random weights, rounded to bfloat16 values; queries and keys loud enough that single keys matter, decays near one."""
    g = torch.Generator().manual_seed(seed)
    w, W = {}, cfg["width"]

    def lin(name, rows, cols, scale=1.0):
        w[name] = torch.randn(rows, cols, generator=g) * scale * cols**-0.5

    def gain(name, n, mean=1.0):
        w[name] = mean + 0.2 * torch.randn(n, generator=g)

    w["embed"] = torch.randn(cfg["vocab"], W, generator=g)
    for i, e in enumerate(cfg["layers"]):
        p, m, x = f"l{i}.", e["mixer"], f"l{i}.mix."
        H, d, vd = m["heads"], m["dim"], m["vdim"]
        for k in ("norm1", "norm1b") + (("norm2", "norm2b") if e["mlp"] else ()):
            gain(p + k, W)
        if e["mlp"]:
            lin(p + "mlp.gate", e["mlp"]["ff"], W, 1.5)
            lin(p + "mlp.up", e["mlp"]["ff"], W, 1.5)
            lin(p + "mlp.down", W, e["mlp"]["ff"])
        lin(x + "o", W, H * vd)
        if e["type"] == "delta":
            G = m["kv_heads"]
            for k, n in (("q", G * d), ("k", G * d), ("v", H * vd)):
                lin(x + k, n, W)
                w[f"{x}{k}.conv"] = torch.randn(n, m["conv"], generator=g) * 0.6
            lin(x + "g", H * vd, W)
            lin(x + "b", H, W)
            lin(x + "a", H, W)
            w[x + "A_log"] = torch.randn(H, generator=g) * 0.5 - 3.0
            w[x + "dt_bias"] = torch.randn(H, generator=g)
            gain(x + "norm", vd)
        elif e["type"] == "latent_attention":
            lin(x + "dq", m["q_rank"], W)
            gain(x + "dq.norm", m["q_rank"])
            lin(x + "uq", H * (d + m["rot_dim"]), m["q_rank"], 1.5)
            lin(x + "dkv", m["kv_rank"] + m["rot_dim"], W, 1.5)
            gain(x + "dkv.norm", m["kv_rank"])
            lin(x + "uk", H * d, m["kv_rank"], 1.5)
            lin(x + "uv", H * vd, m["kv_rank"])
            lin(x + "g", H, W)
        else:
            G = m["kv_heads"]
            lin(x + "q", H * d, W, 1.5)
            lin(x + "k", G * d, W, 1.5)
            lin(x + "v", G * vd, W)
            lin(x + "g", H * vd, W)
            w[x + "vmix"] = torch.tensor(0.3 + 0.1 * i)
    gain("final.norm", W)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


_CACHE = {}


def model(name):
    if name not in _CACHE:
        cfg = dict(CONFIGS[name], architecture="Fifotar")
        _CACHE[name] = (cfg, make_weights(cfg))
    return _CACHE[name]


def oracle_logits(name, toks):
    key = (name, tuple(toks))
    if key not in _CACHE:
        cfg, w = model(name)
        _CACHE[key] = oracle.forward(cfg, {k: v.double() for k, v in w.items()}, list(toks))[0]
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
    """A step of several chunks and row blocks, single tokens and short portions of other requests beside it."""
    seqs = [tokens_of("mixed", n, 70 + n) for n in (150, 9, 12, 20)]
    steps = [[(1, 8, 0), (2, 11, 0)], [(3, 17, 0), (0, 120, 0), (1, 1, 8), (2, 1, 11)], [(3, 3, 17), (0, 30, 120)]]
    got = feed(engine("mixed", run, blocks=18), seqs, steps)
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
    lg, _ = eng.put([9], [torch.tensor(s[:1])], capture_latents=False)  # one token on a slot and pages full of old rows
    check_logits(lg, oracle_logits(name, s)[:1], run[1])


def test_long_decoding(run):
    """Many single tokens, past every chunk, across pages; the batch's other sequence is at another position."""
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


def test_evict_and_restore(run):
    """Cached rows come back from the latents, recurrent states from the host copy of the slot."""
    eng = engine("mixed", run, blocks=8)
    m = eng.model()
    assert m.row_widths == [4 * 40, 2 * 40, 48, 2 * 56, 48, 2 * 32]
    assert m.state_floats() == (4 * 16 * 24 + 3 * (64 + 96)) + (2 * 32 * 16 + 4 * (128 + 32))
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
    assert ((lg.max(-1).values - picked) <= (1e-3 if run[1] == torch.float32 else 0.5)).all()
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
    close(got, oracle_logits("mixed", s), torch.float32, f32=0.15)


def _tp_config():
    return dict(CONFIGS["mixed"], architecture="Fifotar",
                layers=[_att(4, 2, 16, 24, 9, _mlp(40)), _del(4, 2, 16, 24, 3, _mlp(72)),
                        _lat(4, 24, 8, 40, 32, 16, _mlp(48)), _att(6, 2, 16, 24, 33), _del(2, 2, 32, 16, 4)])


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
    from hcache_deepspeed_amd.ops import build, gemv, latent_attention, output_norm, paged
    cls = transformer_class(spec_from_hf(model("mixed")[0]))
    have = ""
    for f in cls.KERNEL_SOURCES:
        with open(os.path.join(build.CSRC, "kernels", f)) as fh:
            have += fh.read()
    used = {"hds_glu_rows"}
    for mod in (delta_op, gemv, latent_attention, output_norm, paged):
        with open(mod.__file__) as fh:
            used |= set(re.findall(r"\)?\.(hds_\w+)\(", fh.read()))
    assert len(used) > 20
    for name in used - {"hds_gemv_recur_bf16"}:
        assert re.search(rf"HDS_EXPORT int {name}\(", have), name


def test_checkpoint_folder_and_registry(tmp_path):
    from safetensors.torch import save_file
    cfg, w = model("first-delta")
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    eng = build_hf_engine(str(tmp_path), {"dtype": "fp32", "state_manager": {"max_context": 64}},
                          device=torch.device("cpu"), num_kv_blocks=4)
    m = eng.model()
    assert m.lm_head is m.embed and len(m.row_widths) == 2
    s = tokens_of("first-delta", 9, 1)
    lg, _ = eng.put([1], [torch.tensor(s)])
    check_logits(lg, oracle_logits("first-delta", s)[-1:], torch.float32)
    mixes = [e["mixer"].get("value_mix") for e in spec_from_hf(model("mixed")[0]).layers]
    assert mixes == [None, None, "source", None, None, "mix", None, "mix"]
    for bad in (dict(cfg["layers"][0], type="other"), dict(cfg["layers"][0], mlp={"kind": "moe"})):
        with pytest.raises(NotImplementedError):
            spec_from_hf(dict(cfg, layers=[bad]))
