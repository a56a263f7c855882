"""Duzizen on the ragged serving engine against the plain implementation in duzizen_oracle.py: every mechanism alone, then
the engine with whole prompts, portions, single tokens, mixed batches, reused pages and slots, decode graphs, eviction, tensor
parallelism, serialization, generation and trace replay. CPU runs use the ops' torch implementations, ``gpu`` runs the HIP
kernels in 32-bit and in bfloat16."""
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
from hcache_deepspeed_amd.inference.v2.modules import (DSExpertLayerConfig, DSGatedMLPConfig, DSLinearConfig, DSMixerConfig,
                                                       instantiate_expert_layer, instantiate_gated_mlp,
                                                       instantiate_linear, instantiate_mixer)
from hcache_deepspeed_amd.ops import matrix_memory as memory_op
from hcache_deepspeed_amd.ops.activations import act_gather
from hcache_deepspeed_amd.ops.experts import ExpertSum, RouterShape, route
from hcache_deepspeed_amd.ops.gemv import gather_gemv
from hcache_deepspeed_amd.ops.head_prep import HeadPrep
from hcache_deepspeed_amd.ops.matrix_memory import MemoryShape, make_memory_plan, matrix_memory, step_ok
from hcache_deepspeed_amd.ops.output_norm import PairSum, embed_pairs, stream_norm
from hcache_deepspeed_amd.ops.paged import HeadShape, head_attention, head_blocks_ok, make_head_plan
from hcache_deepspeed_amd.ops.rope import rope_inv_freq, rope_tables

from . import duzizen_oracle as oracle
from .serving_utils import GPU, Pages, close, feed, portions, rnd, run, tokens  # noqa: F401

# -----------------------------------------------------------------------------------------------
# matrix memories
# -----------------------------------------------------------------------------------------------
# (heads, dim, vdim, rotated): sizes of the vector and matrix-core kernels and of the plain ones
MEMORIES = {"odd": (3, 6, 7, 4), "odd-key": (2, 9, 12, 6), "small": (2, 16, 24, 16), "one": (1, 8, 8, 2),
            "partly": (2, 32, 40, 12), "wide-value": (2, 24, 136, 24), "square": (2, 128, 128, 128),
            "key-72": (3, 72, 40, 40), "plain-key": (1, 160, 48, 96), "value-256": (1, 64, 256, 64),
            "value-300": (1, 40, 300, 8)}
KINDS = ("gated", "fixed", "gated-rotated", "fixed-plain")


def _memory(name, kind, gate=None):
    H, d, e, rot = MEMORIES[name]
    gated = kind.startswith("gated")
    rot = rot if kind in ("fixed", "gated-rotated") else 0
    sh = MemoryShape(H, d, e, 1e-4, gate or ("sigmoid" if gated else "silu"), gated, 9.0 if gated else 0.0, rot)
    return sh, {"dims": rot, "base": 500.0}


def _memory_weights(sh, seed=0):
    """Decays near one, so that early tokens still count at the end; gates over a wide range."""
    w = {"norm": 1 + 0.3 * rnd(sh.heads * sh.vdim, seed=seed)}
    if sh.gated:
        w["i.b"], w["f.b"] = rnd(sh.heads, seed=seed + 1), 4 + rnd(sh.heads, seed=seed + 2)
    else:
        w["norm"] = None
        w["log_decay"] = torch.log(1 - 0.5**(3.0 + torch.arange(sh.heads, dtype=torch.float64)))
    return {k: None if v is None else v.float().double() for k, v in w.items()}


def _memory_oracle(sh, rot, proj, w):
    """The oracle's scans on projected rows."""
    H, d, e, T = sh.heads, sh.dim, sh.vdim, proj.shape[0]
    q, k, v, g, i, f = proj[:, :sh.width].split([H * d, H * d, H * e, H * e] + ([H, H] if sh.gated else [0, 0]), 1)
    q, k, v = q.reshape(T, H, d), k.reshape(T, H, d), v.reshape(T, H, e)
    if sh.rot:
        q, k = (oracle.rotate(x, rot, "interleaved") for x in (q, k))
    if sh.gated:
        i = sh.cap * torch.tanh((i + w["i.b"]) / sh.cap)
        f = oracle.log_sigmoid(sh.cap * torch.tanh((f + w["f.b"]) / sh.cap))
        o = oracle.mlstm_scan(q * d**-0.5, k, v, i, f)
    else:
        o = oracle.retention_scan(q, k * d**-0.5, v, w["log_decay"].exp())
    o = oracle.rms(o, sh.eps).reshape(T, H * e) * (1.0 if w["norm"] is None else w["norm"])
    return o * (oracle.silu(g) if sh.gate == "silu" else oracle.sigmoid(g))


def _projs(sh, lengths, dtype, seed=0):
    out = []
    for n in lengths:
        x = rnd(n, sh.width, seed=seed + n)
        if sh.gated:
            x[:, sh.main_width:] *= 3.0
        out.append(x.to(dtype).double())
    return out


def _run_memory(sh, rot, projs, w, sizes, dev, dtype, serial_max=None, monkeypatch=None, offset=8, slots=None):
    """The op over portions of several sequences, on states full of old values; returns every sequence's outputs."""
    if serial_max is not None:
        monkeypatch.setattr(memory_op, "SERIAL_MAX", serial_max)
    n = len(projs)
    pages = Pages(n, n, 16, 8, slots or list(range(n))[::-1], dev, dtype)
    state = torch.full((n + 1, offset + -(-sh.state_floats // 4) * 4 + 4), 3.0, device=dev)
    f = {k: None if v is None else v.float().to(dev) for k, v in w.items()}
    tables = rope_tables(1024, sh.rot, rot["base"], device=dev) if sh.rot else None
    ld = -(-sh.width // 8) * 8
    single = dev.type == "cuda" and step_ok(sh)
    outs = [[] for _ in projs]
    for step in portions([p.shape[0] for p in projs], sizes):
        b = pages.batch(step)
        x = torch.full((b.current_tokens, ld), float("nan"), dtype=dtype, device=dev)
        x[:, :sh.width] = torch.cat([projs[s][p:p + k] for s, k, p in step]).to(dtype).to(dev)
        out = torch.zeros(b.current_tokens, sh.heads * sh.vdim + 8, dtype=dtype, device=dev)
        plan = make_memory_plan(b.seq_meta_host, b.current_sequences, b.max_new, single, dev)
        matrix_memory(x, sh, f, tables, state, offset, b, plan, out[:, :sh.heads * sh.vdim])
        assert (out[:, sh.heads * sh.vdim:] == 0).all() and (state[n] == 3.0).all()
        assert (state[:, :offset] == 3.0).all() and (state[:, -4:] == 3.0).all()
        for i, (s, k, _) in enumerate(step):
            q0 = b.seq_meta_host[i][0]
            outs[s].append(out[q0:q0 + k, :sh.heads * sh.vdim].double().cpu())
    return [torch.cat(o) for o in outs]


@pytest.mark.parametrize("name", list(MEMORIES))
@pytest.mark.parametrize("kind", KINDS)
@pytest.mark.parametrize("sizes", [[1000], [1], [2], [37, 1, 5, 2, 64, 90]])
def test_matrix_memory(run, name, kind, sizes):
    dev, dtype = run
    sh, rot = _memory(name, kind)
    w, projs = _memory_weights(sh), _projs(sh, (75, 2, 41), dtype)
    got = _run_memory(sh, rot, projs, w, sizes, dev, dtype)
    for g, x in zip(got, projs):
        close(g, _memory_oracle(sh, rot, x, w), dtype, f32=5e-5, bf16=1e-2)


@pytest.mark.parametrize("name", ["small", "square", "key-72", "wide-value", "value-256"])
@pytest.mark.parametrize("kind", KINDS)
@pytest.mark.parametrize("sizes", [[1000], [63, 64, 65], [130, 1, 17]])
def test_matrix_memory_long_portions(run, name, kind, sizes):
    """Several chunks of the matrix-core scan, ends inside and at the edges of chunks."""
    dev, dtype = run
    if dev.type == "cpu":
        pytest.skip("the CPU implementation has one form")
    sh, rot = _memory(name, kind, gate="silu")
    w, projs = _memory_weights(sh, seed=5), _projs(sh, (200, 128, 129), dtype, seed=9)
    got = _run_memory(sh, rot, projs, w, sizes, dev, dtype)
    for g, x in zip(got, projs):
        close(g, _memory_oracle(sh, rot, x, w), dtype, f32=5e-5, bf16=1e-2)


@GPU
@pytest.mark.parametrize("name", ["small", "square", "key-72", "value-256", "partly"])
@pytest.mark.parametrize("kind", KINDS)
def test_chunk_scan_is_the_serial_scan(name, kind, monkeypatch):
    """Both forms keep 32-bit states and 32-bit rotated keys: from the same bfloat16 rows they differ by 32-bit rounding,
    before the outputs are rounded (nearly all outputs are the same bfloat16 number)."""
    dev, dtype = torch.device("cuda"), torch.bfloat16
    print(f"chunk / serial {name} {kind}", flush=True)
    sh, rot = _memory(name, kind)
    w, projs = _memory_weights(sh, seed=9), _projs(sh, (150, 77), dtype, seed=3)
    a = _run_memory(sh, rot, projs, w, [1000], dev, dtype, serial_max=0, monkeypatch=monkeypatch)
    b = _run_memory(sh, rot, projs, w, [1000], dev, dtype, serial_max=10**6, monkeypatch=monkeypatch)
    for x, y in zip(a, b):
        assert ((x - y).abs() <= 0.008 * x.abs() + 1e-4 * x.abs().mean()).all()  # one step of bfloat16
        assert (x != y).double().mean() < 0.01


def test_written_values_are_read_back(run):
    """A value under a key of its own comes back by that key at any distance (input gate open at two tokens only, forget
    gate open); the later write of the same key outweighs the first by its gate."""
    dev, dtype = run
    H, d, e, n = 2, 8, 8, 150
    sh = MemoryShape(H, d, e, 1e-6, "sigmoid", True, 12.0)
    w = {"norm": torch.ones(H * e).double(), "i.b": torch.zeros(H).double(), "f.b": torch.zeros(H).double()}
    x = torch.zeros(n, sh.width, dtype=torch.float64)
    q, k, v, g, i, f = x.split([H * d, H * d, H * e, H * e, H, H], 1)
    q[:, ::d] = 30.0
    k[:, 1::d] = 1.0
    k[3], k[70] = 0.0, 0.0
    k[3, ::d] = k[70, ::d] = 1.0
    v[:] = rnd(n, H * e, seed=1)
    g[:], f[:], i[:] = 8.0, 60.0, -60.0
    i[3], i[70] = 0.0, 60.0
    for sizes in ([1000], [1], [66, 1, 2]):
        (got, ) = _run_memory(sh, None, [x.to(dtype).double()], w, sizes, dev, dtype)
        for lo, hi, src in ((3, 70, 3), (70, n, 70)):
            want = oracle.rms(v[src].to(dtype).double().view(H, e), 1e-6)
            for t in range(lo, hi):
                assert (got[t].view(H, e) - want).abs().max() < 0.05, (sizes, t)


def test_normalizer_floor(run):
    """Queries so small that the floor of the normalizer, e^(-m) + 1e-6, divides: with a maximum near 15 the constant weighs
    more than e^(-m), and less and less as the maximum decays. The head norm's eps is large, so that the size shows."""
    dev, dtype = run
    H, d, e, n, eps = 1, 8, 8, 90, 1e-2
    sh = MemoryShape(H, d, e, eps, "sigmoid", True, 15.0)
    w = {"norm": torch.ones(e).double(), "i.b": torch.zeros(1).double(), "f.b": torch.zeros(1).double()}
    x = rnd(n, sh.width, seed=3)
    x[:, :d] *= 1e-7
    x[:, sh.main_width:] = torch.tensor([-60.0, 2.0], dtype=torch.float64)
    x[0, sh.main_width] = x[40, sh.main_width] = 60.0
    x = x.to(dtype).double()
    want = _memory_oracle(sh, None, x, w)
    # the planted mistake: a normalizer without its constant, that is, read-outs larger by (e^(-m) + 1e-6) / e^(-m)
    f = math.log(1 / (1 + math.exp(-15 * math.tanh(2 / 15))))
    m = torch.tensor([15 * math.tanh(4.0) + f * (t % 40 if t < 80 else t - 40) for t in range(n)], dtype=torch.float64)
    s = torch.sigmoid(x[:, 3 * d:4 * d])
    o = want / s
    size = (o * o).mean(-1, keepdim=True)
    wrong = s * oracle.rms(o * torch.sqrt(eps / (1 - size)) * (1 + 1e-6 * torch.exp(m))[:, None], eps)
    assert ((wrong - want).norm(dim=-1) / want.norm(dim=-1))[[0, 1, 40, 41]].min() > 0.05
    for sizes in ([1000], [1], [2], [17, 1]):
        (got, ) = _run_memory(sh, None, [x], w, sizes, dev, dtype)
        close(got, want, dtype, f32=5e-5, bf16=1e-2)


def test_fixed_decay_powers(run):
    """One written value, then empty keys: what is read is the value times a power of the head's decay, far out too. The head
    norm's eps is large against it, so that the size of the read-out shows."""
    dev, dtype = run
    H, d, e, n = 3, 8, 8, 300
    decay = torch.tensor([0.9, 0.99, 1.0], dtype=torch.float64)
    sh = MemoryShape(H, d, e, 4.0, "silu", False)
    x = torch.zeros(n, sh.width, dtype=torch.float64)
    q, k, v, g = x.split([H * d, H * d, H * e, H * e], 1)
    q[:, ::d], k[0, ::d], g[:] = 1.0, 1.0, 20.0
    v[0] = rnd(H * e, seed=1).to(torch.bfloat16).double()
    w = {"norm": None, "log_decay": decay.log()}
    want = torch.stack([oracle.rms(v[0].view(H, e) * (decay**t)[:, None] * d**-0.5, 4.0).reshape(-1) * 20 for t in range(n)])
    for sizes in ([1000], [1], [129, 2, 40]):
        (got, ) = _run_memory(sh, None, [x], w, sizes, dev, dtype)
        rel = ((got - want).view(n, H, e).norm(dim=-1) / want.view(n, H, e).norm(dim=-1)).max()
        assert rel < (2e-5 if dtype == torch.float32 else 6e-3), (sizes, rel)


# -----------------------------------------------------------------------------------------------
# attention with convolutions, norms across heads, rotation, keys as values, window with kept tokens, zero sink
# -----------------------------------------------------------------------------------------------
@pytest.mark.parametrize("n,base,sc", [(24, 500.0, None), (32, 10000.0, (8.0, 1.0, 4.0, 512)), (10, 100.0, (3.0, 0.5, 2.0, 64)),
                                       (2, 7.0, (2.0, 1.0, 2.0, 16)), (64, 1e6, (16.0, 1.0, 8.0, 100000))])
def test_frequencies(n, base, sc):
    rot, ours = {"dims": n, "base": base}, None
    if sc:
        rot["scaling"] = dict(zip(("factor", "low", "high", "original"), sc))
        ours = {"rope_type": "llama3", "factor": sc[0], "low_freq_factor": sc[1], "high_freq_factor": sc[2],
                "original_max_position_embeddings": sc[3]}
    want = torch.tensor(oracle.frequencies(rot), dtype=torch.float64)
    assert torch.allclose(rope_inv_freq(n, base, ours), want, rtol=1e-12)
    cos, sin = rope_tables(3000, n, base, ours)
    assert torch.allclose(cos[2999].double(), (2999 * want).cos(), atol=1e-6)
    assert torch.allclose(sin[2999].double(), (2999 * want).sin(), atol=1e-6)


# (heads, kv heads, dim, rotated, taps, window, kept)
HEADS = {"one": (1, 1, 8, 8, 1, 0, 0), "odd": (3, 1, 6, 4, 3, 9, 2), "group": (4, 2, 24, 8, 4, 16, 5),
         "all-rotated": (6, 3, 32, 32, 2, 33, 17), "no-kept": (4, 4, 40, 20, 5, 12, 0), "kept-wide": (2, 1, 128, 64, 3, 20, 40),
         "big-group": (10, 2, 16, 6, 9, 40, 3), "wide": (8, 2, 264, 32, 2, 30, 4), "one-back": (4, 2, 48, 16, 4, 1, 1)}


def _heads(name, **other):
    H, G, d, rot, taps, window, keep = HEADS[name]
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": d, "conv": taps, "scale": 1.3 * d**-0.5,
         "rot": {"dims": rot, "base": 300.0, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 128}},
         "mask": {"size": window, "keep_first": keep} if window else None}
    sh = HeadShape(heads=H, kv_heads=G, dim=d, vdim=d, window=window, keep=keep, scale=m["scale"], eps=1e-4, gated=False,
                   prep=True, taps=taps, rot=rot, shared=True, **other)
    return sh, m


def _head_weights(sh, seed=0):
    H, G, d = sh.heads, sh.kv_heads, sh.dim
    p = {"q.conv": rnd(H * d, sh.taps, seed=seed, scale=0.8), "k.conv": rnd(G * d, sh.taps, seed=seed + 1, scale=0.8),
         "q.norm": 1.5 + 0.3 * rnd(H * d, seed=seed + 2), "k.norm": 1.5 + 0.3 * rnd(G * d, seed=seed + 3)}
    p = {k: v.float().double() for k, v in p.items()}
    parts = torch.eye(sh.channels, dtype=torch.float64).split([H * d, G * d])
    return dict(p, q=parts[0], k=parts[1], o=torch.eye(H * d).double())


def _run_heads(sh, m, projs, p, sizes, dev, dtype, block_size=16):
    n = len(projs)
    per = -(-max(x.shape[0] for x in projs) // block_size)
    pages = Pages(n, n * per, block_size, sh.row, list(range(n))[::-1], dev, dtype)
    offset = 4
    state = torch.full((n + 1, offset + -(-sh.state_floats // 4) * 4 + 4), 3.0, device=dev)
    sc = m["rot"].get("scaling")
    ours = sc and {"rope_type": "llama3", "factor": sc["factor"], "low_freq_factor": sc["low"],
                   "high_freq_factor": sc["high"], "original_max_position_embeddings": sc["original"]}
    f = {k: p[k].float().to(dev).contiguous() for k in ("q.norm", "k.norm")}
    conv = torch.cat([p["q.conv"], p["k.conv"]]).float().t().contiguous().to(dev)
    prep = HeadPrep(conv, f["q.norm"], f["k.norm"], rope_tables(1024, sh.rot, m["rot"]["base"], ours, device=dev), state,
                    offset)
    sink = torch.zeros(sh.heads, device=dev)
    ld = -(-sh.channels // 8) * 8
    blocks = dev.type == "cuda" and head_blocks_ok(sh, dtype)
    outs = [[] for _ in projs]
    for step in portions([x.shape[0] for x in projs], sizes):
        b = pages.batch(step)
        T = b.current_tokens
        x = torch.full((T, ld), float("nan"), dtype=dtype, device=dev)
        x[:, :sh.channels] = torch.cat([projs[s][q:q + k] for s, k, q in step]).to(dtype).to(dev)
        out = torch.zeros(T, sh.heads * sh.vdim + 8, dtype=dtype, device=dev)
        plan = make_head_plan(b.seq_meta_host, T, sh.heads, sh.kv_heads, blocks and b.max_new > 1, dev)
        head_attention(x, sh, None, None, sink, pages.cache, b, plan, out[:, :sh.heads * sh.vdim], prep=prep)
        assert (out[:, sh.heads * sh.vdim:] == 0).all() and (state[n] == 3.0).all()
        assert (state[:, :offset] == 3.0).all() and (state[:, -4:] == 3.0).all()
        for i, (s, k, _) in enumerate(step):
            q0 = b.seq_meta_host[i][0]
            outs[s].append(out[q0:q0 + k, :sh.heads * sh.vdim].double().cpu())
    return [torch.cat(o) for o in outs]


@pytest.mark.parametrize("name", list(HEADS))
@pytest.mark.parametrize("sizes", [[1000], [1], [2], [37, 1, 5, 2, 64, 90]])
def test_attention(run, name, sizes):
    dev, dtype = run
    sh, m = _heads(name)
    p = _head_weights(sh)
    projs = [rnd(n, sh.channels, seed=40 + n).to(dtype).double() for n in (90, 2, 41)]
    got = _run_heads(sh, m, projs, p, sizes, dev, dtype)
    for g, x in zip(got, projs):
        close(g, oracle.attention(x, p, m, sh.eps), dtype, f32=5e-5, bf16=3e-2)


@pytest.mark.parametrize("window,keep,loud", [(64, 0, 20), (64, 16, 15), (64, 16, 16), (33, 70, 69), (33, 70, 70), (100, 3, 0),
                                              (16, 64, 63), (16, 64, 64), (65, 1, 130)])
@pytest.mark.parametrize("sizes", [[300], [1], [131, 2, 17]])
def test_one_key_inside_and_outside_the_window(run, window, keep, loud, sizes):
    """One key's score towers over the others': a query gives back its value exactly while it is in the window or among the
    kept first tokens, in prompts and in decoding, at page borders and next to them."""
    dev, dtype = run
    H, G, d, n = 4, 2, 16, 300
    sh = HeadShape(heads=H, kv_heads=G, dim=d, vdim=d, window=window, keep=keep, scale=1.0, eps=1e-6, gated=False, prep=True,
                   taps=2, rot=4, shared=True)
    m = {"rot": {"dims": 4, "base": 100.0}}
    x = torch.zeros(n, sh.channels, dtype=torch.float64)
    q, k = x.split([H * d, G * d], 1)
    q[:, 8::d] = 10.0            # (not rotated)
    k[:] = 0.3 * rnd(n, G * d, seed=loud)
    k[:, 8::d] = 0.0
    k[loud] = 0.0
    k[loud, 8::d], k[loud, 9::d] = 20.0, 8.0
    p = {"q.conv": torch.tensor([[0.0, 1.0]]).double().expand(H * d, 2), "q.norm": torch.full((H * d, ), 2.0).double(),
         "k.conv": torch.tensor([[0.0, 1.0]]).double().expand(G * d, 2), "k.norm": torch.full((G * d, ), 2.0).double()}
    got, = _run_heads(sh, m, [x.to(dtype).double()], p, sizes, dev, dtype)
    value = torch.zeros(H, d, dtype=torch.float64)
    value[:, 8], value[:, 9] = 20.0, 8.0
    for i in range(n):
        same = float((got[i].view(H, d) - value).norm() / value.norm()) < 0.05
        assert same == (i >= loud and (i - loud < window or loud < keep)), (i, same)


def test_sink_takes_its_share(run):
    """Keys of score zero: n visible ones share n / (n + 1) of the weight."""
    dev, dtype = run
    sh, m = _heads("one-back")
    m = dict(m, mask={"size": 7, "keep_first": 2})
    sh = HeadShape(**{**sh.__dict__, "window": 7, "keep": 2})
    p = _head_weights(sh)
    p["q.norm"] = torch.zeros_like(p["q.norm"])
    x = rnd(30, sh.channels, seed=1).to(dtype).double()
    got, = _run_heads(sh, m, [x], p, [30], dev, dtype)
    u = oracle.short_conv(x[:, 4 * 48:], p["k.conv"]).view(30, 2, 48)
    for i in range(30):
        js = [j for j in range(i + 1) if i - j < 7 or j < 2]
        want = (u[js].sum(0) / (len(js) + 1)).repeat_interleave(2, 0).reshape(1, -1)
        close(got[i:i + 1], want, dtype, bf16=2e-2)


def test_convolution_crosses_portions(run):
    """An impulse shows in exactly the next taps - 1 tokens, wherever the portions are cut."""
    dev, dtype = run
    sh = HeadShape(heads=1, kv_heads=1, dim=8, vdim=8, window=1, keep=0, scale=0.0, eps=1e-6, gated=False, prep=True, taps=4,
                   rot=2, shared=True)  # every token sees itself with half the weight: outputs are v / 2
    cw = torch.tensor([[0.5, -2.0, 4.0, 1.0]]).double().expand(8, 4)
    p = {"q.conv": cw, "k.conv": cw, "q.norm": torch.ones(8).double(), "k.norm": torch.ones(8).double()}
    for at in (0, 3, 15, 16, 17):
        x = torch.zeros(24, 16, dtype=torch.float64)
        x[at] = 1.0
        for sizes in ([24], [1], [2], [3, 1, 5]):
            got, = _run_heads(sh, {"rot": {"dims": 2, "base": 9.0}}, [x], p, sizes, dev, dtype)
            want = torch.zeros(24, 8, dtype=torch.float64)
            for back, c in enumerate((1.0, 4.0, -2.0, 0.5)):
                if at + back < 24:
                    want[at + back] = c / 2
            assert torch.allclose(got, want, atol=1e-6), (at, sizes)


# -----------------------------------------------------------------------------------------------
# both mixers as registered modules
# -----------------------------------------------------------------------------------------------
def _mixer(kind, params, W, dev, dtype, weights, eps=1e-4):
    """The registered mixer with its linears and its weights on the device."""
    mix = instantiate_mixer(DSMixerConfig(kind, W, params, eps, 1, dtype))
    mix.bind_positions(512, dev)
    lins = {k: instantiate_linear(DSLinearConfig(*io)) for k, io in
            {"in.w": (W, mix.in_width), "out.w": (mix.out_width, W), **mix.extra_linears()}.items()}
    raw = mix.shard(weights, lambda t: t, lambda t: t)
    raw["out.w"] = raw.pop("o.w", None)
    w = {k: None if v is None else v.to(dtype if k.endswith((".w", "o.w")) and "conv" not in k else torch.float32)
         .contiguous().to(dev) for k, v in raw.items()}
    return mix, lins, w


def _run_mixer(kind, m, p, W, dev, dtype, sizes, eps, result, lengths=(75, 2, 41)):
    cfg = _config([{"type": kind, "mixer": m, "mlp": None}], width=W, norm={"eps": eps})
    mix, lins, w = _mixer(kind, spec_from_hf(cfg).layers[0]["mixer"], W, dev, dtype, p, eps)
    xs = [rnd(n, W, seed=20 + n).to(dtype).double() for n in lengths]
    pages = Pages(3, 18, 16, max(mix.cache_row, 1), [2, 0, 1], dev, dtype)
    state = torch.full((3, 8 + mix.state_floats()), 3.0, device=dev)
    outs = [[] for _ in xs]
    for step in portions([x.shape[0] for x in xs], sizes):
        b = pages.batch(step)
        x = torch.cat([xs[s][q:q + n] for s, n, q in step]).to(dtype).to(dev)
        mid = torch.zeros(b.current_tokens, mix.out_width, dtype=dtype, device=dev)
        mix(x, w, lins, mid, b, pages.cache, state, 8)
        y = result(mix.output(mid, w, lins, lambda t: t))
        for i, (s, n, _) in enumerate(step):
            q0 = b.seq_meta_host[i][0]
            outs[s].append(y[q0:q0 + n].double().cpu())
    return xs, [torch.cat(o) for o in outs]


def _config(layers, **other):
    return dict(dict(architecture="Duzizen", vocab=31, width=40, norm={"eps": 1e-5}, token_side={"dim": 8},
                     embedding={"bigram": {"buckets": 53, "mul_prev": 7, "mul_cur": 3}}, layers=layers), **other)


def _mls(H, d, e, cap=8.0, mlp=None):
    return {"type": "mlstm", "mixer": {"heads": H, "dim": d, "vdim": e, "gate_cap": cap}, "mlp": mlp}


def _par(left, right, mlp=None, base=400.0, sc=(4.0, 1.0, 4.0, 64), scale=1.5, decay=None):
    """left: (heads, kv heads, dim, rotated, taps, window, kept); right: (heads, dim, vdim, rotated)"""
    H, G, d, rot, taps, window, keep = left
    RH, rd, re_, rr = right
    scaling = dict(zip(("factor", "low", "high", "original"), sc)) if sc else None
    return {"type": "parallel", "mlp": mlp,
            "mixer": {"left": {"heads": H, "kv_heads": G, "dim": d, "vdim": d, "conv": taps, "scale": scale * d**-0.5,
                               "mask": {"size": window, "keep_first": keep}, "rot": {"dims": rot, "base": base,
                                                                                     "scaling": scaling}},
                      "right": {"heads": RH, "dim": rd, "vdim": re_, "rot": {"dims": rr, "base": 50 * base},
                                "decay": decay or [1 - 0.5**(3 + 2 * h) for h in range(RH)]}}}


def _mixer_weights(m, W, kind, seed=0):
    """Random weights of a mixer, rounded to bfloat16 values. The memories' keys resemble their queries: where the products
    of a first token's query and key cancel, its read-out (a value, normed per head) would turn with their sign."""
    g = torch.Generator().manual_seed(seed)
    p = {}

    def lin(name, rows, cols, scale=1.0):
        p[name] = torch.randn(rows, cols, generator=g) * scale * cols**-0.5

    def gain(name, n, mean=1.0):
        p[name] = mean + 0.2 * torch.randn(n, generator=g)

    if kind == "mlstm":
        H, d, e = m["heads"], m["dim"], m["vdim"]
        for k, n in (("q", H * d), ("k", H * d), ("v", H * e), ("g", H * e)):
            lin(k, n, W)
        p["k"] = 0.8 * p["q"] + 0.6 * p["k"]
        lin("o", W, H * e)
        gain("norm", H * e)
        lin("i", H, W)
        lin("f", H, W)
        gain("i.b", H, 0.5)
        gain("f.b", H, 3.5)
        return {k: v.to(torch.bfloat16) for k, v in p.items()}
    a, r = m["left"], m["right"]
    for k, n in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"])):
        lin(f"left.{k}", n, W)
        gain(f"left.{k}.norm", n, 1.3)
        p[f"left.{k}.conv"] = torch.randn(n, a["conv"], generator=g) * 0.7
    lin("left.o", W, a["heads"] * a["dim"])
    for k, n in (("q", r["heads"] * r["dim"]), ("k", r["heads"] * r["dim"]), ("v", r["heads"] * r["vdim"]),
                 ("g", r["heads"] * r["vdim"])):
        lin(f"right.{k}", n, W)
    p["right.k"] = 0.8 * p["right.q"] + 0.6 * p["right.k"]
    lin("right.o", W, r["heads"] * r["vdim"])
    gain("left.out", W)
    gain("right.out", W)
    return {k: v.to(torch.bfloat16) for k, v in p.items()}


MIXERS = {"mlstm": _mls(3, 24, 16), "mlstm-odd": _mls(2, 5, 7, 3.0),
          "parallel": _par((4, 2, 24, 8, 3, 20, 6), (3, 16, 24, 12)),
          "parallel-odd": _par((3, 1, 6, 4, 2, 9, 3), (2, 10, 5, 6), sc=None),
          "parallel-wide": _par((8, 2, 64, 64, 4, 30, 40), (2, 128, 64, 128))}


@pytest.mark.parametrize("name", list(MIXERS))
@pytest.mark.parametrize("sizes", [[1000], [1], [2], [37, 1, 5, 2, 64, 90]])
def test_mixers(run, name, sizes):
    """The mixers from their input rows to the output projection: both rotation layouts, norms of both sides."""
    dev, dtype = run
    e, W, eps = MIXERS[name], 40, 1e-4
    p = _mixer_weights(e["mixer"], W, e["type"], seed=3)
    xs, got = _run_mixer(e["type"], e["mixer"], p, W, dev, dtype, sizes, eps,
                         lambda y: y.total(eps) if isinstance(y, PairSum) else y)
    f = {k: v.double() for k, v in p.items()}
    for g, x in zip(got, xs):
        want = (oracle.mlstm if e["type"] == "mlstm" else oracle.parallel)(x, f, e["mixer"], eps)
        close(g, want, dtype, f32=5e-5, bf16=4e-2)


# -----------------------------------------------------------------------------------------------
# norms, embedding, per-layer input, feed-forward
# -----------------------------------------------------------------------------------------------
STREAMS = [(5, 64), (1, 37), (3, 2048), (100, 72), (2, 4104), (70, 1536), (1, 9000), (80, 4096), (65, 37), (3, 320), (1, 8192)]


def _gains(W, seed):
    return [(m + 0.4 * rnd(W, seed=seed + i)).float().double() for i, m in enumerate((1.0, 0.0))]


@pytest.mark.parametrize("T,W", STREAMS)
@pytest.mark.parametrize("kind", ["plain", "pair", "experts", "none"])
def test_stream_norm(run, T, W, kind):
    dev, dtype = run
    eps = 1e-3
    f = lambda t: t.float().to(dev)  # noqa: E731
    a = lambda t: t.to(dtype).to(dev)  # noqa: E731
    x = rnd(T, W, seed=1, scale=3.0).float().double() + 5.0  # far from mean zero
    g, b = _gains(W, 3)
    gn, bn = _gains(W, 5)
    d1, d2 = ((rnd(T, W, seed=s, scale=0.1) + 0.3).to(dtype).double() for s in (11, 12))
    if kind == "plain":
        delta, total = a(d1), d1
    elif kind == "pair":
        ga, gb = _gains(W, 7)
        delta = PairSum(a(d1), a(d2), f(ga), f(gb))
        total = (oracle.rms(d1, eps, ga) + oracle.rms(d2, eps, gb)) / 2
    elif kind == "experts":
        y = torch.cat([d1, d2]).to(dtype)
        row = torch.randperm(2 * T, generator=torch.Generator().manual_seed(T)).view(T, 2).to(torch.int32)
        delta = ExpertSum(a(y), torch.zeros(T, 2, dtype=torch.int32, device=dev), None, row.to(dev), 3)
        total = y.double()[row.long()].sum(1)
    else:
        delta = total = None
    want = x if total is None else x + oracle.layer_norm(total, eps, g, b)
    pad = 1 if dtype == torch.float32 else 128
    x1, y = stream_norm(f(x), delta, (f(g), f(b)), (f(gn), f(bn)), eps, dtype, pad=pad)
    close(x1, want, torch.float32)
    close(y[:, :W], oracle.layer_norm(want, eps, gn, bn), dtype, bf16=5e-3)
    assert y.shape[1] % pad == 0 and (y[:, W:] == 0).all()
    x1, y = stream_norm(f(x), delta, (f(g), f(b)), None, eps, dtype)
    close(x1, want, torch.float32)
    close(y, want, dtype, bf16=5e-3)
    if kind != "pair":
        want = x if total is None else x + oracle.rms(total, eps, g)
    idx = torch.tensor([T - 1, 0], dtype=torch.int32, device=dev)
    none, y = stream_norm(f(x), delta, f(g) if kind != "pair" else (f(g), f(b)), f(gn), eps, dtype, idx=idx)
    assert none is None
    close(y, oracle.rms(want, eps, gn)[[T - 1, 0]], dtype, bf16=5e-3)


@pytest.mark.parametrize("W,buckets,mp,mc", [(64, 101, 31, 7), (37, 13, 1, 1), (136, 64, 100003, 65537)])
@pytest.mark.parametrize("sizes", [[1000], [1], [2], [9, 1, 3]])
def test_pair_embedding(run, W, buckets, mp, mc, sizes):
    """The previous token crosses the steps; slots full of old values do not show at a sequence's start."""
    dev, dtype = run
    V = 50
    embed, pairs = rnd(V, W, seed=1).to(dtype), rnd(buckets + 1, W, seed=2).to(dtype)
    seqs = [tokens(V, n, n) for n in (23, 1, 12)]
    pages = Pages(3, 6, 16, 8, [2, 0, 1], dev, dtype)
    state = torch.full((3, 12), 7.0, device=dev)
    outs = [[] for _ in seqs]
    for step in portions([len(s) for s in seqs], sizes):
        b = pages.batch(step)
        ids = torch.tensor([t for s, n, q in step for t in seqs[s][q:q + n]], device=dev)
        x = embed_pairs(embed.to(dev), pairs.to(dev), ids, 1.0, mp, mc, state, 4, b)
        assert (state[:, :4] == 7.0).all() and (state[:, 5:] == 7.0).all()
        for i, (s, n, _) in enumerate(step):
            q0 = b.seq_meta_host[i][0]
            outs[s].append(x[q0:q0 + n].double().cpu())
    for s, o in zip(seqs, outs):
        want = oracle.embedding(s, embed.double(), pairs.double(), {"mul_prev": mp, "mul_cur": mc})
        close(torch.cat(o), want, torch.float32, f32=1e-6)


@pytest.mark.parametrize("T,C,layers", [(5, 24, 3), (1, 8, 1), (130, 37, 2), (3, 256, 4)])
def test_act_gather(run, T, C, layers):
    dev, dtype = run
    x, table = rnd(T, C + 8, seed=1).to(dtype), rnd(19, layers * C, seed=2).to(dtype)
    ids = torch.randint(0, 19, (T, ), generator=torch.Generator().manual_seed(3))
    for i in range(layers):
        got = act_gather(x.to(dev)[:, :C], "gelu_tanh", table.to(dev)[:, i * C:(i + 1) * C], ids.to(dev))
        want = oracle.gelu(x[:, :C].double()) * table[ids, i * C:(i + 1) * C].double()
        close(got, want, dtype, bf16=5e-3)


@GPU
@pytest.mark.parametrize("M,W,C", [(1, 40, 24), (1, 4096, 256), (2, 128, 5), (7, 256, 40), (16, 1024, 72)])
def test_gather_gemv(M, W, C):
    """The product of decode rows with the activation and the table's row in one kernel: the same numbers as the two."""
    print(f"gather {M} {W} {C}", flush=True)
    x, w = (rnd(n, W, seed=s, scale=W**-0.25).to(torch.bfloat16).cuda() for n, s in ((M, 1), (C, 2)))
    table = rnd(19, 3 * C, seed=3).to(torch.bfloat16).cuda()[:, C:2 * C]
    ids = torch.randint(0, 19, (M, ), generator=torch.Generator().manual_seed(3))
    got = gather_gemv(x, w, "gelu_tanh", table, ids.cuda())
    want = oracle.gelu(x.double().cpu() @ w.double().cpu().T) * table.double().cpu()[ids]
    close(got, want, torch.bfloat16, bf16=1e-2)
    assert gather_gemv(x.float(), w.float(), "gelu_tanh", table.float(), ids.cuda()) is None


@pytest.mark.parametrize("T", [1, 2, 40])
@pytest.mark.parametrize("W,ff", [(64, 48), (40, 37), (128, 256)])
def test_dense_feed_forward(run, T, W, ff):
    dev, dtype = run
    p = {k: rnd(ff, W, seed=s, scale=2 * W**-0.5).to(dtype).double() for k, s in (("gate", 1), ("up", 2))}
    x = rnd(T, W, seed=3).to(dtype).double()
    mlp = instantiate_gated_mlp(DSGatedMLPConfig(W, ff, "gelu_tanh"))
    out = torch.zeros(T, ff, dtype=dtype, device=dev)
    mlp(x.to(dtype).to(dev), torch.cat([p["gate"], p["up"]]).to(dtype).to(dev),
        instantiate_linear(DSLinearConfig(W, 2 * ff)), out)
    close(out, oracle.dense(x, dict(p, down=torch.eye(ff).double())), dtype, bf16=2e-2)


@pytest.mark.parametrize("E,top", [(1, 1), (12, 1), (64, 6), (100, 7), (200, 3)])
def test_sigmoid_router(run, E, top):
    dev, dtype = run
    if dtype == torch.bfloat16:
        pytest.skip("router logits are 32-bit")
    z = rnd(70, E, seed=E, scale=2.0).float()
    expert, weight = route(z.to(dev), None, RouterShape(E, top=top, score="sigmoid", weigh_input=True))
    s = oracle.sigmoid(z.double())
    best = torch.sort(s, -1, descending=True)
    assert torch.equal(expert.cpu().long(), best.indices[:, :top])
    close(weight, best.values[:, :top], torch.float32)


@pytest.mark.parametrize("E,top,W,ff,limit", [(5, 2, 40, 24, 0.7), (12, 1, 64, 48, 2.0), (3, 3, 37, 11, 1.0),
                                              (9, 4, 256, 128, 50.0), (1, 1, 24, 8, 0.5)])
@pytest.mark.parametrize("T", [1, 7, 64, 65, 300])
def test_experts_with_weighed_inputs(run, E, top, W, ff, limit, T):
    dev, dtype = run
    p = {"router": rnd(E, W, seed=1, scale=2 * W**-0.5)}
    for e in range(E):
        p.update({f"e{e}.gate": rnd(ff, W, seed=10 * e + 2, scale=3 * W**-0.5),
                  f"e{e}.up": rnd(ff, W, seed=10 * e + 3, scale=3 * W**-0.5),
                  f"e{e}.down": rnd(W, ff, seed=10 * e + 4, scale=ff**-0.5)})
    p = {k: v.to(torch.bfloat16).double() for k, v in p.items()}
    x = rnd(T, W, seed=5).to(dtype).double()
    if dtype == torch.bfloat16:  # no close calls: a tie may fall either way
        s = torch.sort(oracle.sigmoid(x @ p["router"].T), -1, descending=True).values
        if top < E:
            x = x[(s[:, top - 1] - s[:, top]) > 1e-4]
    layer = instantiate_expert_layer(DSExpertLayerConfig(W, ff, RouterShape(E, top=top, score="sigmoid", weigh_input=True),
                                                         input_dtype=dtype, activation="clamped", limit=limit))
    stack = {k: torch.stack([p[f"e{e}.{k}"] for e in range(E)]) for k in ("gate", "up", "down")}
    raw = layer.shard(dict(stack, router=p["router"]), lambda t: t, lambda t: t)
    w = {k: None if v is None else v.to(dtype).contiguous().to(dev) for k, v in raw.items()}
    rows = torch.zeros(x.shape[0], -(-W // layer.row_pad()) * layer.row_pad(), dtype=dtype, device=dev)
    rows[:, :W] = x.to(dtype).to(dev)
    parts = layer(rows, w)
    got = layer.total(torch.zeros(x.shape[0], W, device=dev), parts)
    want = oracle.experts(x, p, {"router": {"top": top}, "expert": {"limit": limit}})
    close(got, want, dtype, f32=5e-5, bf16=2e-2)
    x1, _ = stream_norm(torch.zeros(x.shape[0], W, device=dev), parts, torch.ones(W, device=dev), None, 1e-3, dtype)
    close(x1, oracle.rms(want, 1e-3), torch.float32, f32=5e-5 if dtype == torch.float32 else 2e-2)


# -----------------------------------------------------------------------------------------------
# models
# -----------------------------------------------------------------------------------------------
def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(E, top, ff, limit=1.5):
    return {"kind": "moe", "router": {"experts": E, "top": top}, "expert": {"ff": ff, "limit": limit}}


CONFIGS = {
    # every pair of neighbours, feed-forwards of both kinds in some layers
    "mixed": _config([_mls(2, 16, 24, 6.0, _dense(40)), _par((4, 2, 24, 8, 3, 13, 5), (3, 16, 24, 12), _moe(6, 2, 24)),
                      _par((2, 2, 32, 32, 4, 40, 18), (2, 32, 16, 32)), _mls(3, 24, 16, 15.0, _moe(4, 1, 40, 0.8)),
                      _par((6, 2, 16, 6, 2, 1, 3), (4, 8, 8, 8), _dense(56), sc=None), _mls(1, 32, 32)],
                     vocab=131, width=64, token_side={"dim": 16}),
    # begins with a parallel layer, one value of everything
    "first-parallel": _config([_par((1, 1, 8, 2, 1, 16, 1), (1, 8, 8, 2), _moe(1, 1, 8, 3.0)), _mls(1, 8, 8, 1.0, _dense(8))],
                              vocab=90, width=48, norm={"eps": 1e-3}, token_side={"dim": 1},
                              embedding={"bigram": {"buckets": 1, "mul_prev": 1, "mul_cur": 1}}),
    "wide": _config([_mls(2, 128, 128, 10.0, _dense(136)), _par((8, 1, 128, 64, 4, 50, 9), (2, 128, 64, 128), _moe(8, 3, 64))],
                    vocab=67, width=128, norm={"eps": 1e-6}, token_side={"dim": 72}),
    # no state but the memories', nothing that can be left out
    "memories": _config([_mls(4, 16, 16, 5.0), _mls(2, 8, 40, 5.0, _moe(3, 3, 16))], vocab=75, width=40),
    # sizes the matrix-core and vector paths do not take
    "odd": _config([_mls(3, 5, 7, 4.0, _moe(5, 2, 11)), _par((3, 1, 6, 4, 3, 12, 4), (2, 10, 5, 6), _dense(13)),
                    _par((2, 1, 10, 10, 2, 5, 2), (1, 3, 9, 2), _moe(2, 1, 7), sc=None)],
                   vocab=61, width=37, token_side={"dim": 5}),
}


def make_weights(cfg, seed=0):
    """Random weights, rounded to bfloat16 values; queries and keys loud enough that single keys matter, decays near one."""
    g = torch.Generator().manual_seed(seed)
    w, W, C = {}, cfg["width"], cfg["token_side"]["dim"]

    def lin(name, rows, cols, scale=1.0):
        w[name] = torch.randn(rows, cols, generator=g) * scale * cols**-0.5

    def norm(name):
        w[name], w[name + ".b"] = 1 + 0.2 * torch.randn(W, generator=g), 0.2 * torch.randn(W, generator=g)

    lin("embed", cfg["vocab"], W, W**0.5)
    lin("head", cfg["vocab"], W)
    lin("bigram", cfg["embedding"]["bigram"]["buckets"] + 1, W, 0.7 * W**0.5)
    lin("side.embed", cfg["vocab"], C * len(cfg["layers"]), (C * len(cfg["layers"]))**0.5)
    norm("final.norm")
    for i, e in enumerate(cfg["layers"]):
        p = f"l{i}."
        for k in ("norm1", "norm1b") + (("norm2", "norm2b") if e["mlp"] else ()):
            norm(p + k)
        for k, v in _mixer_weights(e["mixer"], W, e["type"], seed=1000 * seed + i).items():
            w[p + "mix." + k] = v
        m = e["mlp"]
        if m and m["kind"] == "dense":
            for k, r, c in (("gate", m["ff"], W), ("up", m["ff"], W), ("down", W, m["ff"])):
                lin(f"{p}mlp.{k}", r, c, 1.3)
        elif m:
            lin(p + "mlp.router", m["router"]["experts"], W, 2.0)
            for x in range(m["router"]["experts"]):
                for k, r, c in (("gate", m["expert"]["ff"], W), ("up", m["expert"]["ff"], W), ("down", W, m["expert"]["ff"])):
                    lin(f"{p}mlp.e{x}.{k}", r, c, 1.5)
        lin(p + "side.gate", C, W)
        lin(p + "side.proj", W, C)
        w[p + "side.norm"] = 0.6 + 0.2 * torch.randn(W, generator=g)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


_CACHE = {}


def _all_chosen(cfg):
    """The same model with every expert chosen: rounding to bfloat16 cannot turn a close call of the router."""
    layers = []
    for e in cfg["layers"]:
        m = e["mlp"]
        if m and m["kind"] == "moe":
            m = dict(m, router={"experts": m["router"]["experts"], "top": m["router"]["experts"]})
        layers.append(dict(e, mlp=m))
    return dict(cfg, layers=layers)


def model(name, dtype=torch.float32):
    key = (name, dtype)
    if key not in _CACHE:
        cfg = CONFIGS[name] if dtype == torch.float32 else _all_chosen(CONFIGS[name])
        _CACHE[key] = (cfg, make_weights(cfg))
    return _CACHE[key]


def oracle_logits(name, toks, dtype):
    key = (name, tuple(toks), dtype)
    if key not in _CACHE:
        cfg, w = model(name, dtype)
        _CACHE[key] = oracle.forward(cfg, {k: v.double() for k, v in w.items()}, list(toks))[0]
    return _CACHE[key]


def engine(name, run, blocks=12, slots=4, block_size=16, max_context=192, **conf):
    dev, dtype = run
    cfg, w = model(name, dtype)
    spec = spec_from_hf(cfg)
    ec = RaggedInferenceEngineConfig.from_dict(dict(
        dtype="fp32" if dtype == torch.float32 else "bf16",
        state_manager=dict(max_context=max_context, max_ragged_batch_size=512, max_tracked_sequences=slots,
                           kv_block_size=block_size), **conf))
    return InferenceEngineV2(spec, convert_hf(w, spec), ec, device=dev, num_kv_blocks=blocks)


def tokens_of(name, n, seed):
    return tokens(CONFIGS[name]["vocab"], n, seed)


def check_logits(got, want, dtype):
    """Nearly all rows to the type's rounding, all of them to a multiple of it: a read-out that cancels nearly to nothing in
    front of a head norm magnifies rounding."""
    got, want = got.double().cpu(), want.double().cpu()
    assert got.shape == want.shape and torch.isfinite(got).all()
    err = (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
    most, worst = (1e-4, 1e-3) if dtype == torch.float32 else (6e-2, 0.3)
    assert (err > most).sum() <= max(1, 0.05 * err.numel()) and err.max() <= worst, err.topk(min(5, err.numel()))


@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("sizes", [[1000], [2], [1], [21, 1, 16, 2, 3, 17]])
def test_portions(run, name, sizes):
    """Whole prompts, portions of several sizes and single tokens give the logits of the whole sequence."""
    eng = engine(name, run)
    toks = tokens_of(name, 61, 1)
    got, = feed(eng, [toks], portions([61], sizes))
    check_logits(got, oracle_logits(name, toks, run[1]), run[1])
    eng.flush(0)
    assert eng.free_blocks == 12


@pytest.mark.parametrize("name", list(CONFIGS))
def test_mixed_batches(run, name):
    """Unequal requests, portions beside single tokens: each gets the logits it gets alone."""
    seqs = [tokens_of(name, n, 10 + n) for n in (50, 1, 23, 37)]
    got = feed(engine(name, run, blocks=16), seqs, portions([len(s) for s in seqs], [19, 1, 1, 2, 30, 1, 5], seed=3))
    for g, s in zip(got, seqs):
        check_logits(g, oracle_logits(name, s, run[1]), run[1])


def test_long_mixed_step(run):
    """A step of several chunks and row blocks, single tokens and short portions of other requests beside it."""
    seqs = [tokens_of("mixed", n, 70 + n) for n in (150, 9, 12, 20)]
    steps = [[(1, 8, 0), (2, 11, 0)], [(3, 17, 0), (0, 120, 0), (1, 1, 8), (2, 1, 11)], [(3, 3, 17), (0, 30, 120)]]
    got = feed(engine("mixed", run, blocks=18), seqs, steps)
    for g, s in zip(got, seqs):
        check_logits(g, oracle_logits("mixed", s, run[1]), run[1])


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
    check_logits(torch.cat(outs), oracle_logits(name, s, run[1]), run[1])
    check_logits(first[1], oracle_logits(name, tokens_of(name, 60, 21), run[1]), run[1])
    eng.flush(5)
    lg, _ = eng.put([9], [torch.tensor(s[:1])], capture_latents=False)  # one token on a slot and pages full of old rows
    check_logits(lg, oracle_logits(name, s, run[1])[:1], run[1])


def test_long_decoding(run):
    """Many single tokens, past every window, across pages; the batch's other sequence is at another position."""
    toks, other = tokens_of("mixed", 130, 30), tokens_of("mixed", 120, 31)
    steps = [[(0, 5, 0)], [(1, 2, 0)]] + [[(0, 1, 5 + i)] + ([(1, 1, 2 + i)] if i < 118 else []) for i in range(125)]
    got = feed(engine("mixed", run, blocks=24), [toks, other], steps)
    check_logits(got[0], oracle_logits("mixed", toks, run[1]), run[1])
    check_logits(got[1], oracle_logits("mixed", other, run[1]), run[1])


def test_wanted_places(run):
    eng = engine("mixed", run)
    a, b = tokens_of("mixed", 30, 1), tokens_of("mixed", 12, 2)
    lg, _ = eng.put(["a", "b"], [torch.tensor(a), torch.tensor(b)], capture_latents=False, logits_at=[[4, 29, 0], []])
    check_logits(lg, oracle_logits("mixed", a, run[1])[[4, 29, 0]], run[1])
    lg, _ = eng.put(["b"], [torch.tensor(b[:1])], capture_latents=False, logits_at=[[]])
    assert lg.shape == (0, 131)


def test_evict_and_restore(run):
    """Cached rows come back from the latents; memories, convolution tails and the last token from the slot's copy."""
    eng = engine("mixed", run, blocks=8)
    m = eng.model()
    assert m.row_widths == [2 * 48, 2 * 64, 2 * 32]
    mem = [2 * (16 * 24 + 16) + 2, 3 * 16 * 24, 2 * 32 * 16, 3 * (24 * 16 + 24) + 3, 4 * 64, 32 * 32 + 32 + 1]
    ring = [3 * 6 * 24, 4 * 4 * 32, 2 * 8 * 16]
    assert m.state_floats() == 4 + sum(-(-n // 4) * 4 for n in mem + ring)
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
    check_logits(torch.cat(got), oracle_logits("mixed", s, run[1])[33:], run[1])


@pytest.mark.parametrize("name", ["mixed", "odd", "memories"])
def test_greedy_generation(run, name):
    """The engine's own generation loop; compared with the plain implementation step by step along its own tokens."""
    prompt = tokens_of(name, 19, 5)
    eng = engine(name, run, blocks=8)
    out = eng.generate(1, torch.tensor(prompt), max_new_tokens=24)
    lg = oracle_logits(name, prompt + out, run[1])[len(prompt) - 1:-1]
    picked = lg[torch.arange(24), out]
    gap = lg.max(-1).values - picked
    if run[1] == torch.float32:
        assert out == lg.argmax(-1).tolist()
    else:
        assert gap.max() < 0.5
    eng.flush(1)
    g = torch.Generator(device=run[0]).manual_seed(0)
    sampled = eng.generate(2, torch.tensor(prompt), max_new_tokens=8, do_sample=True, temperature=0.7, top_k=5,
                           generator=g)
    lg = oracle_logits(name, prompt + sampled, run[1])[len(prompt) - 1:-1]
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
        check_logits(outs[True][:, i], oracle_logits("mixed", s, torch.bfloat16)[11 + i % 3:17 + i % 3], torch.bfloat16)


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
    want = oracle_logits("mixed", s, torch.float32)
    err = (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
    assert err.median() < 0.1 and (err > 0.3).sum() <= 3


def _tp_config():
    return _config([_mls(2, 16, 24, 6.0, _dense(40)), _par((4, 2, 24, 8, 3, 13, 5), (4, 16, 24, 12), _moe(6, 2, 24)),
                    _par((2, 2, 32, 32, 1, 40, 18), (2, 32, 16, 32)), _mls(4, 24, 16, 15.0, _moe(4, 1, 40, 0.8))],
                   vocab=131, width=64, token_side={"dim": 16})


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


@GPU
@pytest.mark.parametrize("name", ["group", "odd"])
def test_norm_sums_of_all_ranks(name):
    """What a rank with half of the heads computes with the other rank's sums of squares is what one with all heads does."""
    dev = torch.device("cuda")
    print(f"rank sums {name}", flush=True)
    sh, m = _heads("group" if name == "group" else "one-back")
    p = _head_weights(sh)
    H, G, d = sh.heads, sh.kv_heads, sh.dim
    x = rnd(21, sh.channels, seed=1).float().double()
    want = oracle.attention(x, p, m, sh.eps)
    half = HeadShape(**{**sh.__dict__, "heads": H // 2, "kv_heads": G // 2})
    rows = [torch.cat([torch.arange(r * H // 2 * d, (r + 1) * H // 2 * d),
                       H * d + torch.arange(r * G // 2 * d, (r + 1) * G // 2 * d)]) for r in (0, 1)]
    u = torch.cat([oracle.short_conv(x[:, :H * d], p["q.conv"]), oracle.short_conv(x[:, H * d:], p["k.conv"])], 1)
    sums = [torch.stack([u[:, r[:H // 2 * d]].pow(2).sum(1), u[:, r[H // 2 * d:]].pow(2).sum(1)], 1) for r in rows]
    sc = m["rot"]["scaling"]
    tables = rope_tables(512, sh.rot, m["rot"]["base"],
                         {"rope_type": "llama3", "factor": sc["factor"], "low_freq_factor": sc["low"],
                          "high_freq_factor": sc["high"], "original_max_position_embeddings": sc["original"]}, device=dev)
    for r in (0, 1):
        pages = Pages(1, 2, 16, half.row, [0], dev, torch.float32)
        state = torch.full((1, half.state_floats), 3.0, device=dev)
        conv = torch.cat([p["q.conv"], p["k.conv"]])[rows[r]].float().t().contiguous().to(dev)
        norms = torch.cat([p["q.norm"], p["k.norm"]])[rows[r]].float().to(dev)

        def total(mine, step):
            assert torch.allclose(mine.double().cpu(), sums[r][step], rtol=1e-5)
            return mine + sums[1 - r][step].float().to(dev)

        outs = []
        for a, n in ((0, 13), (13, 1), (14, 7)):
            b = pages.batch([(0, n, a)])
            prep = HeadPrep(conv, norms[:H // 2 * d].contiguous(), norms[H // 2 * d:].contiguous(), tables, state, 0, 2,
                            lambda t: total(t, slice(a, a + n)))
            out = torch.zeros(n, H // 2 * d, device=dev)
            head_attention(x[a:a + n, rows[r]].float().to(dev), half, None, None, torch.zeros(H // 2, device=dev), pages.cache, b,
                           make_head_plan(b.seq_meta_host, n, H // 2, G // 2, False, dev), out, prep=prep)
            outs.append(out.double().cpu())
        close(torch.cat(outs), want[:, r * H // 2 * d:(r + 1) * H // 2 * d], torch.float32, f32=5e-5)


def test_trace_replay(run, tmp_path):
    """The trace runner's step function and the checkpoint folder it reads."""
    from safetensors.torch import save_file

    from hcache_deepspeed_amd.inference.v2 import trace
    cfg, w = model("mixed", run[1])
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

    check_logits(read(0), oracle_logits("mixed", a, run[1])[[0, 7]], run[1])
    want = torch.stack([oracle_logits("mixed", b + [3], run[1])[70], oracle_logits("mixed", a, run[1])[30]])
    check_logits(read(2), want, run[1])
    check_logits(read(3), oracle_logits("mixed", a, run[1])[:1], run[1])


def test_kernel_sources_of_the_model_class_are_complete():
    """A library of the class's KERNEL_SOURCES alone exports every entry point its ops call."""
    from hcache_deepspeed_amd.ops import activations, build, experts, gemv, output_norm, paged
    cls = transformer_class(spec_from_hf(model("mixed")[0]))
    have = ""
    for f in cls.KERNEL_SOURCES:
        with open(os.path.join(build.CSRC, "kernels", f)) as fh:
            have += fh.read()
    used = set()
    for mod in (memory_op, activations, experts, gemv, output_norm, paged):
        with open(mod.__file__) as fh:
            used |= set(re.findall(r"\)?\.(hds_\w+)\(", fh.read()))
    assert len(used) > 20
    for name in used:
        assert re.search(rf"HDS_EXPORT int {name}\(", have), name


def test_checkpoint_folder_and_registry(tmp_path):
    from safetensors.torch import save_file
    cfg, w = model("first-parallel")
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    eng = build_hf_engine(str(tmp_path), {"dtype": "fp32", "state_manager": {"max_context": 64}},
                          device=torch.device("cpu"), num_kv_blocks=4)
    s = tokens_of("first-parallel", 9, 1)
    lg, _ = eng.put([1], [torch.tensor(s)])
    check_logits(lg, oracle_logits("first-parallel", s, torch.float32)[-1:], torch.float32)
    layers = spec_from_hf(model("mixed")[0]).layers
    assert [e["mixer"]["type"] for e in layers] == ["mlstm", "parallel", "parallel", "mlstm", "parallel", "mlstm"]
    assert layers[1]["mixer"]["left"]["keep"] == 5 and layers[3]["mixer"]["cap"] == 15.0
    for bad in (dict(cfg["layers"][0], type="other"), dict(cfg["layers"][0], mlp={"kind": "other"})):
        with pytest.raises(NotImplementedError):
            spec_from_hf(dict(cfg, layers=[bad]))
    left = dict(cfg["layers"][0]["mixer"]["left"], vdim=16)
    with pytest.raises(ValueError):
        spec_from_hf(dict(cfg, layers=[dict(cfg["layers"][0], mixer=dict(cfg["layers"][0]["mixer"], left=left))]))
