"""From the q / k / v projection to paged attention (csrc/kernels/head_prep.hip): short causal convolutions of q and k, RMS
norms over all heads of q (of k), rotation of neighbouring pairs, and the cache append, in one kernel. ``ops.paged.HeadShape``
says which of them a layer has; the keys as they leave the convolution may serve as the values.

CPU tensors take a plain torch form.
"""
from dataclasses import dataclass
from typing import Optional

import torch

from . import native
from .paged import copy_rows


@dataclass
class HeadPrep:
    """What ``head_prep`` works with. conv: [taps, channels] float32, the last row is the current token's, or None; norms:
    [heads * dim] and [kv_heads * dim] float32, or None; tables: (cos, sin) [positions, rot / 2] or None;
    ``state[slot, offset:]`` is read and advanced. total: sums the rows' sums of squares [T, 2] over the ranks that share the
    heads, which hold ``ranks`` times as many."""
    conv: Optional[torch.Tensor]
    q_norm: Optional[torch.Tensor]
    k_norm: Optional[torch.Tensor]
    tables: Optional[tuple]
    state: Optional[torch.Tensor]
    offset: int
    ranks: int = 1
    total: Optional[callable] = None


def head_prep(x, shape, p, cache, batch):
    """x: [T, >= shape.qkv_width] projection, q heads | k heads (| v heads). Appends the step's keys and values to ``cache``
    and returns the queries [T, heads * dim]."""
    sh, T = shape, x.shape[0]
    if not native.use_native(x):
        return _head_prep_cpu(x, sh, p, cache, batch)
    lib, dev = native.kernels(), x.device
    cos, sin = p.tables if sh.rot else (None, None)
    assert x.stride(1) == 1 and cache.dtype == x.dtype and cache.shape[2] == sh.row and x.shape[1] >= sh.qkv_width
    assert sh.taps == 1 or (p.state is not None and p.offset + sh.state_floats <= p.state.shape[1])
    assert p.conv is None or (p.conv.shape == (sh.taps, sh.channels) and p.conv.is_contiguous())
    assert p.q_norm is None or (p.q_norm.numel() == sh.heads * sh.dim and p.k_norm.numel() == sh.kv_heads * sh.dim)
    assert not sh.rot or cos.shape[1] == sh.rot // 2
    q = torch.empty(T, sh.heads * sh.dim, dtype=x.dtype, device=dev)
    tab = batch.block_tables

    def run(out, sums):
        native.check(
            lib.hds_head_prep(native.dt(x), x.data_ptr(), x.stride(0), sh.heads, sh.kv_heads, sh.dim, sh.vdim, sh.taps,
                              sh.rot, int(sh.shared), native.ptr(p.conv), native.ptr(p.q_norm), native.ptr(p.k_norm),
                              native.ptr(cos), native.ptr(sin), q.data_ptr(), q.stride(0), cache.data_ptr(),
                              tab.data_ptr(), tab.shape[1], cache.shape[1], batch.tok_seq.data_ptr(),
                              batch.tok_pos.data_ptr(), batch.seq_meta.data_ptr(),
                              None if p.state is None else p.state.data_ptr() + 4 * p.offset,
                              0 if p.state is None else p.state.stride(0), batch.slots.data_ptr(), native.ptr(out),
                              native.ptr(sums), p.ranks * sh.heads * sh.dim, p.ranks * sh.kv_heads * sh.dim,
                              float(sh.eps), T, batch.current_sequences, batch.max_new, native.stream()), "head_prep")

    sums = None
    if p.ranks > 1 and p.q_norm is not None:
        sums = torch.empty(T, 2, dtype=torch.float32, device=dev)
        run(sums, None)
        sums = p.total(sums)
    run(None, sums)
    return q


def _head_prep_cpu(x, sh, p, cache, batch):
    T, C, taps = x.shape[0], sh.channels, sh.taps
    u = x[:, :C].float()
    if p.conv is not None:
        raw, u = u, torch.zeros(T, C)
        for s, (q0, n, seen) in enumerate(batch.seq_meta_host):
            ring = None
            if taps > 1:
                ring = p.state[batch.slots_host[s], p.offset:p.offset + sh.state_floats].view(taps, C)
            for t in range(n):
                pos = seen + t
                if ring is None:
                    u[q0 + t] = p.conv[0] * raw[q0 + t]
                    continue
                ring[pos % taps] = raw[q0 + t]
                u[q0 + t] = sum(p.conv[taps - 1 - k] * ring[(pos - k) % taps] for k in range(min(taps, pos + 1)))
    q, k = u.split([sh.heads * sh.dim, sh.kv_heads * sh.dim], 1)
    v = k if sh.shared else x[:, C:sh.qkv_width].float()
    if p.q_norm is not None:
        sums = torch.stack([(q * q).sum(1), (k * k).sum(1)], 1)
        if p.ranks > 1:
            sums = p.total(sums)
        q, k = (a / torch.sqrt(sums[:, j:j + 1] / (p.ranks * a.shape[1]) + sh.eps) * w
                for j, (a, w) in enumerate(((q, p.q_norm), (k, p.k_norm))))
    if sh.rot:
        pos, h = batch.tok_pos.long(), sh.rot // 2
        c, s = (t[pos][:, None, :h] for t in p.tables)

        def turned(a):
            a = a.reshape(T, -1, sh.dim).clone()
            x0, x1 = a[..., 0:sh.rot:2].clone(), a[..., 1:sh.rot:2].clone()
            a[..., 0:sh.rot:2], a[..., 1:sh.rot:2] = x0 * c - x1 * s, x1 * c + x0 * s
            return a.reshape(T, -1)

        q, k = turned(q), turned(k)
    copy_rows(cache, torch.cat([k, v], 1), batch.tok_seq, batch.tok_pos, batch.block_tables, to_cache=True)
    return q.to(x.dtype)
