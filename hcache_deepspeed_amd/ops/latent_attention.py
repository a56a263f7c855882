"""Latent (compressed K/V) attention over a paged cache of latent rows (HIP, csrc/kernels/latent_attn.hip).

The cache of a layer is [blocks, block_size, rank + rot]: the normed latent and the rotated shared key part. A batch is
split by sequence (``plan``): single tokens and short portions run *absorbed* on the cached rows, longer portions
*expanded* (keys and values of all heads from one matrix product over the gathered visible rows, then an MFMA flash
kernel). CPU tensors run the torch implementation below."""
from dataclasses import dataclass
from typing import Optional

import numpy as np
import torch
import torch.nn.functional as F

from . import native
from .paged import copy_rows


@dataclass(frozen=True)
class LatentShape:
    heads: int
    dim: int        # unrotated query / key dims of a head
    rot: int        # rotated dims (shared key part)
    rot_dims: int   # of those, how many turn
    rank: int
    vdim: int
    window: int     # 0: every earlier token
    scale: float
    eps: float
    gated: bool = False  # a gate per token and head multiplies the head's output

    @property
    def row(self):
        return self.rank + self.rot

    @property
    def q_width(self):
        return self.heads * (self.dim + self.rot)


# Portions of at most this many tokens run absorbed: each re-reads the visible rows, which costs less than expanding them
# once (a product over the whole window) up to some twenty tokens
ABSORB_MAX = 16


@dataclass
class LatentPlan:
    """Which tokens of a step run absorbed and where the expanded sequences' rows lie in their gathered matrix."""
    n_abs: int
    atok: Optional[torch.Tensor] = None     # None: every token, in order
    n_pre: int = 0
    max_pre: int = 0
    ws_rows: int = 0
    meta: Optional[torch.Tensor] = None     # [n_pre, 4] q_start, n_new, first ws row, keys before the new ones
    ws_row: Optional[torch.Tensor] = None   # [T]
    g_seq: Optional[torch.Tensor] = None    # gathered (past) rows: sequence, position, ws row
    g_pos: Optional[torch.Tensor] = None
    g_dst: Optional[torch.Tensor] = None


def can_expand(shape, dtype):
    return dtype == torch.bfloat16 and bool(
        native.kernels().hds_latent_prefill_ok(shape.dim, shape.rot, shape.rank, shape.vdim))


def make_plan(seq_meta_host, n_tokens, window, expand, device, absorb_max=None):
    """The plan of one batch for attention layers with this window; one host-to-device copy, shared by the layers."""
    absorb_max = ABSORB_MAX if absorb_max is None else absorb_max
    if not expand or all(n <= absorb_max for (_, n, _) in seq_meta_host):
        return LatentPlan(n_abs=n_tokens)
    atok, meta, gs, gp, gd = [], [], [], [], []
    ws_row = np.full(n_tokens, -1, dtype=np.int32)
    rows = 0
    for s, (q0, n, seen) in enumerate(seq_meta_host):
        if n <= absorb_max:
            atok.append(np.arange(q0, q0 + n, dtype=np.int32))
            continue
        past = min(seen, window - 1) if window > 0 else seen
        meta.append((q0, n, rows, past))
        gs.append(np.full(past, s, dtype=np.int32))
        gp.append(np.arange(seen - past, seen, dtype=np.int32))
        gd.append(np.arange(rows, rows + past, dtype=np.int32))
        ws_row[q0:q0 + n] = np.arange(rows + past, rows + past + n, dtype=np.int32)
        rows += past + n
    parts = [np.asarray(meta, dtype=np.int32).ravel(), ws_row,
             np.concatenate(atok) if atok else np.empty(0, np.int32)] + [np.concatenate(a) for a in (gs, gp, gd)]
    flat = np.concatenate(parts)
    host = torch.empty(flat.size, dtype=torch.int32, pin_memory=device.type == "cuda")
    host.numpy()[:] = flat
    dev = host.to(device, non_blocking=True)
    views, o = [], 0
    for a in parts:
        views.append(dev[o:o + a.size])
        o += a.size
    plan = LatentPlan(n_abs=parts[2].size, atok=views[2], n_pre=len(meta), max_pre=max(x[1] for x in meta),
                      ws_rows=rows, meta=views[0].view(-1, 4), ws_row=views[1], g_seq=views[3], g_pos=views[4],
                      g_dst=views[5])
    plan._keep = host  # pinned source of an asynchronous copy
    return plan


def _rot(v, cos, sin, rdims):
    """v [..., rot] float32 with cos / sin [..., rdims / 2]: interleaved pairs of the first rdims turn."""
    a, b = v[..., 0:rdims:2], v[..., 1:rdims:2]
    out = v.clone()
    out[..., 0:rdims:2] = a * cos - b * sin
    out[..., 1:rdims:2] = b * cos + a * sin
    return out


def latent_attention(q, ckr, shape, norm_w, uk, uv, ukv, cos, sin, cache, batch, plan, out, gate=None):
    """q: [T, q_width] projected query heads (consumed); ckr: [T, rank + rot] latent and shared key part. norm_w: [rank]
    float32; uk: [H, dim, rank]; uv: [H, vdim, rank]; ukv: the two stacked, [H (dim + vdim), rank]; gate: [T, H] or None.
    Appends the step's rows to ``cache`` and writes the heads' values into ``out`` [T, H vdim] (unit column strides)."""
    assert (gate is not None) == shape.gated
    if not native.use_native(q):
        return _latent_attention_cpu(q, ckr, shape, norm_w, uk, uv, cos, sin, cache, batch, out, gate)
    sh, lib = shape, native.kernels()
    T, dt, dev = q.shape[0], native.dt(q), q.device
    H, bs, mb = sh.heads, cache.shape[1], batch.block_tables.shape[1]
    assert q.stride(1) == 1 and ckr.stride(1) == 1 and out.stride(1) == 1
    assert cache.dtype == q.dtype == out.dtype == ckr.dtype and q.shape[1] == sh.q_width and ckr.shape[1] == sh.row
    assert gate is None or (gate.dtype == q.dtype and gate.shape == (T, H) and gate.stride(1) == 1)
    gp, ldg = native.ptr(gate), 0 if gate is None else gate.stride(0)
    assert cache.shape[2] == sh.row and cos.shape[1] == sh.rot_dims // 2
    n_abs = plan.n_abs
    qa = torch.empty(n_abs, H, sh.row, dtype=q.dtype, device=dev) if n_abs else None
    ws = torch.empty(plan.ws_rows, sh.row, dtype=q.dtype, device=dev) if plan.n_pre else None
    native.check(
        lib.hds_latent_prep(dt, q.data_ptr(), q.stride(0), ckr.data_ptr(), ckr.stride(0), norm_w.data_ptr(),
                            cos.data_ptr(), sin.data_ptr(), cache.data_ptr(), batch.tok_seq.data_ptr(), batch.tok_pos.data_ptr(),
                            batch.block_tables.data_ptr(), native.ptr(plan.ws_row), native.ptr(ws), uk.data_ptr(),
                            native.ptr(plan.atok), native.ptr(qa), T, n_abs, cos.shape[0], mb, bs, H, sh.dim, sh.rot,
                            sh.rot_dims, sh.rank, float(sh.eps), native.stream()), "latent_prep")
    if n_abs:
        mfma = int(q.dtype == torch.bfloat16 and bool(lib.hds_latent_decode_mfma_ok(sh.rank, sh.rot)))
        cap = mb * bs
        keys = min(cap, sh.window) if sh.window else cap
        splits = lib.hds_latent_decode_splits(n_abs, H, sh.rank, sh.rot, mfma, keys)
        part_o = torch.empty(n_abs * H * splits * sh.rank, dtype=torch.float32, device=dev)
        part_ml = torch.empty(n_abs * H * splits * 2, dtype=torch.float32, device=dev)
        native.check(
            lib.hds_latent_decode(dt, qa.data_ptr(), cache.data_ptr(), part_o.data_ptr(), part_ml.data_ptr(),
                                  native.ptr(plan.atok), batch.tok_seq.data_ptr(), batch.tok_pos.data_ptr(),
                                  batch.block_tables.data_ptr(), mb, bs, n_abs, H, sh.rank, sh.rot, splits, sh.window,
                                  float(sh.scale), mfma, native.stream()), "latent_decode")
        native.check(
            lib.hds_latent_combine(dt, part_o.data_ptr(), part_ml.data_ptr(), uv.data_ptr(), native.ptr(plan.atok),
                                   out.data_ptr(), out.stride(0), gp, ldg, n_abs, H, sh.rank, sh.vdim, splits,
                                   native.stream()), "latent_combine")
    if plan.n_pre:
        copy_rows(cache, ws, plan.g_seq, plan.g_pos, batch.block_tables, plan.g_dst)
        kv = F.linear(ws[:, :sh.rank], ukv)
        kr = ws[:, sh.rank:]
        o = out if out.stride(0) % 8 == 0 and out.data_ptr() % 16 == 0 else \
            torch.empty(T, out.shape[1], dtype=out.dtype, device=dev)
        if q.stride(0) % 8 or q.data_ptr() % 16:
            q = q.clone(memory_format=torch.contiguous_format)
        native.check(
            lib.hds_latent_prefill(q.data_ptr(), q.stride(0), kv.data_ptr(), kv.stride(0), kr.data_ptr(),
                                   kr.stride(0), o.data_ptr(), o.stride(0), gp, ldg, plan.meta.data_ptr(), plan.n_pre,
                                   plan.max_pre, H, sh.dim, sh.rot, sh.rank, sh.vdim, sh.window, float(sh.scale),
                                   native.stream()), "latent_prefill")
        if o is not out:
            rows = (plan.ws_row >= 0)[:, None]
            out.copy_(torch.where(rows, o, out))
    return out


def _latent_attention_cpu(q, ckr, sh, norm_w, uk, uv, cos, sin, cache, batch, out, gate):
    H, dh, T = sh.heads, sh.dim + sh.rot, q.shape[0]
    pos = batch.tok_pos.long()
    q = q.float().reshape(T, H, dh)
    c, kr = ckr.float().split([sh.rank, sh.rot], 1)
    c = c / torch.sqrt((c * c).mean(-1, keepdim=True) + sh.eps) * norm_w
    row = torch.cat([c, _rot(kr, cos[pos], sin[pos], sh.rot_dims)], 1).to(cache.dtype)
    copy_rows(cache, row, batch.tok_seq, batch.tok_pos, batch.block_tables, to_cache=True)
    qr = _rot(q[..., sh.dim:], cos[pos][:, None], sin[pos][:, None], sh.rot_dims)
    qa = torch.cat([torch.einsum("thd,hdr->thr", q[..., :sh.dim], uk.float()), qr], -1)
    bs = cache.shape[1]
    for s, (q0, n, seen) in enumerate(batch.seq_meta_host):
        if n == 0:
            continue
        lo = max(0, seen - sh.window + 1) if sh.window else 0
        j = torch.arange(lo, seen + n)
        blk = batch.block_tables[s, j // bs].long()
        k = cache[blk, j % bs].float()
        sc = torch.einsum("thr,jr->htj", qa[q0:q0 + n], k) * sh.scale
        i = seen + torch.arange(n)
        hide = j[None] > i[:, None]
        if sh.window:
            hide |= j[None] <= i[:, None] - sh.window
        p = torch.softmax(sc.masked_fill(hide[None], float("-inf")), -1)
        o = torch.einsum("htj,jr->thr", p, k[:, :sh.rank])
        o = torch.einsum("thr,hvr->thv", o, uv.float())
        if gate is not None:
            o = o * torch.sigmoid(gate[q0:q0 + n].float())[..., None]
        out[q0:q0 + n] = o.reshape(n, -1).to(out.dtype)
    return out
