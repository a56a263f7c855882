"""Paged-KV serving ops: fused RoPE + KV scatter, ragged paged attention (HIP, csrc/kernels/paged_attn.hip), and
``head_attention``: attention with heads that are normed one by one and not rotated, or convolved, normed across the heads
and rotated (ops/head_prep.py), with a window (and first tokens that stay visible) or chunks, a soft cap, a sink,
value mixing and an output gate over the same kernels.

Reference parity: inference/v2/kernels/ragged_ops/linear_blocked_kv_rotary (``LinearBlockedKVCopy``,
``BlockedRotaryEmbeddings``) and ragged_ops/blocked_flash (``BlockedFlashAttn``) + atom_builder.
CPU tensors run torch references (used by the CPU test-suite and as the GPU numerics oracle).
"""
from dataclasses import dataclass
from typing import Optional

import torch

from . import native

ROWS_PER_ATOM = 128


def kernel_head_dim_ok(D):
    """The HIP serving kernels are instantiated for the same head dims as the training FlashAttention."""
    from .attention import head_dim_supported
    return head_dim_supported(D)


def kv_rope_scatter(qkv, cache, tok_seq, tok_pos, block_tables, cos, sin, n_q, n_kv, rotate_q=True, do_rope=True,
                    rotary_dim=0):
    """qkv: [T, n_q + 2 n_kv, D]; cache: [num_blocks, block_size, 2, n_kv, D] (one layer).

    RoPE at absolute positions ``tok_pos`` on q (in place, if ``rotate_q``) and k (the first ``rotary_dim``
    dims only when 0 < rotary_dim < D: partial rotary of Phi / GPT-NeoX style models); k and v are written
    to ``cache[block_tables[tok_seq[t], pos // bs], pos % bs]``.
    """
    T, NH, D = qkv.shape
    bs = cache.shape[1]
    partial = do_rope and 0 < rotary_dim < D
    if native.use_native(qkv):
        rd = rotary_dim if partial else D
        if D % 4 or rd % 8:
            raise NotImplementedError(f"kv_rope_scatter: head_dim {D} / rotary_dim {rd} not supported on the GPU")
        native.check(
            native.kernels().hds_kv_rope_scatter(native.dt(qkv), qkv.data_ptr(), qkv.stride(0), cache.data_ptr(),
                                                 tok_seq.data_ptr(), tok_pos.data_ptr(), block_tables.data_ptr(),
                                                 block_tables.shape[1], cos.data_ptr() if do_rope else None,
                                                 sin.data_ptr() if do_rope else None, T, n_q, n_kv, D, rd, bs,
                                                 int(rotate_q), int(do_rope), native.stream()), "kv_rope_scatter")
        return
    pos = tok_pos.long()
    rd = rotary_dim if partial else D
    half = rd // 2

    def rot(x):
        if not do_rope:
            return x
        c = cos[pos][:, None, :half]
        s = sin[pos][:, None, :half]
        xf = x[..., :rd].float()
        a, b = xf[..., :half], xf[..., half:]
        r = torch.cat([a * c - b * s, b * c + a * s], -1).to(x.dtype)
        return torch.cat([r, x[..., rd:]], -1) if rd < D else r

    if rotate_q:
        qkv[:, :n_q] = rot(qkv[:, :n_q])
    k = rot(qkv[:, n_q:n_q + n_kv])
    v = qkv[:, n_q + n_kv:]
    blk = block_tables[tok_seq.long(), pos // bs].long()
    slot = pos % bs
    cache[blk, slot, 0] = k
    cache[blk, slot, 1] = v


def build_atoms(seq_meta_host, n_q, n_kv):
    """seq_meta_host: list of (q_start, n_new, seen). Returns int32 [n_atoms, 3] = (seq, kv_head, row_start)."""
    G = n_q // n_kv
    atoms = []
    for s, (_, n_new, _) in enumerate(seq_meta_host):
        rows = n_new * G
        for hk in range(n_kv):
            for r0 in range(0, rows, ROWS_PER_ATOM):
                atoms.append((s, hk, r0))
    return torch.tensor(atoms if atoms else [(0, 0, 0)], dtype=torch.int32), len(atoms)


_COUNTERS = {}
_MERGE_IN_KERNEL = __import__("os").environ.get("HDS_DECODE_MERGE_IN_KERNEL", "0") == "1"


def _merge_counters(device, n):
    """Per-device ints the split-K decode kernel counts finished splits in (the last workgroup of a (sequence, kv
    head) merges the splits and zeroes its counter again): allocated once, zeroed, with room for 64K (sequence, kv
    head) pairs, so a HIP-graph decode captures a stable address. ``HDS_DECODE_MERGE_IN_KERNEL=1`` turns it on;
    by default the separate combine launch merges: the device-scope release each split workgroup needs (its L2
    written back for the other XCDs) cost more than the saved launch -- v2 decode B = 1 200 vs 247 tok/s, B = 8
    1,096 vs 1,490 (profiles/r6/decode_merge/)."""
    if not _MERGE_IN_KERNEL or n > 65536:
        return None
    buf = _COUNTERS.get(device)
    if buf is None:
        buf = _COUNTERS[device] = torch.zeros(65536, dtype=torch.int32, device=device)
    return buf.data_ptr()


def paged_attention(q, cache, atoms, n_atoms, seq_meta, block_tables, n_q, n_kv, scale, window=0,
                    seq_meta_host=None, block_tables_host=None, decode=False):
    """q: [T, n_q, D] (token-strided view ok). Returns o [T, n_q, D]. ``decode``: every sequence of the batch has
    exactly one new token (T == n_seqs) -- the split-K paged decode kernel runs instead of the atom kernel; its key
    splits are sized from the cache capacity (block table width x block size), so one launch shape serves every
    step of a HIP-graph decode."""
    T, _, D = q.shape
    o = torch.empty(T, n_q, D, device=q.device, dtype=q.dtype)
    if native.use_native(q):
        if not kernel_head_dim_ok(D) or q.dtype != torch.bfloat16:
            raise NotImplementedError(f"paged_attention: head_dim {D} / {q.dtype} has no HIP kernel")
        lib = native.kernels()
        if decode:
            n_seqs = T
            keys = block_tables.shape[1] * cache.shape[1]
            splits = lib.hds_paged_decode_splits(n_seqs, n_kv, min(keys, window) if window else keys)
            part_o = part_ml = None
            if splits > 1:
                part_o = torch.empty(n_seqs * n_q * splits * D, device=q.device, dtype=torch.float32)
                part_ml = torch.empty(n_seqs * n_q * splits * 2, device=q.device, dtype=torch.float32)
            counters = _merge_counters(q.device, n_seqs * n_kv) if splits > 1 and n_q // n_kv <= 8 else None
            native.check(
                lib.hds_paged_decode(native.dt(q), 0, q.data_ptr(), q.stride(0), cache.data_ptr(), o.data_ptr(),
                                     n_q * D, native.ptr(part_o), native.ptr(part_ml), seq_meta.data_ptr(), None, None,
                                     None, block_tables.data_ptr(), block_tables.shape[1], cache.shape[1], n_seqs, n_q,
                                     n_kv, D, D, splits, float(scale), int(window), 0, 0, 0.0, None, None, 0, 1, counters,
                                     native.stream()), "paged_decode")
            return o
        native.check(
            lib.hds_paged_attn(q.data_ptr(), q.stride(0), cache.data_ptr(), o.data_ptr(), n_q * D, atoms.data_ptr(),
                               n_atoms, seq_meta.data_ptr(), block_tables.data_ptr(), block_tables.shape[1],
                               cache.shape[1], n_q, n_kv, D, D, float(scale), int(window), 0, 0, 0.0, None, None, 0, 1,
                               native.stream()), "paged_attn")
        return o
    meta = seq_meta_host if seq_meta_host is not None else seq_meta.tolist()
    tables = block_tables_host if block_tables_host is not None else block_tables
    bs = cache.shape[1]
    G = n_q // n_kv
    for s, (q0, n_new, seen) in enumerate(meta):
        if n_new == 0:
            continue
        ctx = seen + n_new
        pos = torch.arange(ctx, device=q.device)
        blk = torch.as_tensor(tables[s], device=q.device)[pos // bs].long()
        kk = cache[blk, pos % bs, 0].float()  # [ctx, n_kv, D]
        vv = cache[blk, pos % bs, 1].float()
        qq = q[q0:q0 + n_new].float()  # [n_new, n_q, D]
        kk = kk.repeat_interleave(G, 1)
        vv = vv.repeat_interleave(G, 1)
        sc = torch.einsum("thd,chd->htc", qq, kk) * scale
        qpos = seen + torch.arange(n_new, device=q.device)
        mask = pos[None, :] > qpos[:, None]
        if window:
            mask |= pos[None, :] <= qpos[:, None] - window
        sc = sc.masked_fill(mask[None], float("-inf"))
        o[q0:q0 + n_new] = torch.einsum("htc,chd->thd", torch.softmax(sc, -1), vv).to(o.dtype)
    return o


def copy_rows(cache, rows, seq, pos, tables, dst_row=None, to_cache=False):
    """Rows of ``cache`` [blocks, block_size, W] at (seq[i], pos[i]) -> ``rows[dst_row[i] or i]``, or back."""
    n, W, bs = seq.numel(), cache.shape[2], cache.shape[1]
    if n == 0:
        return
    if native.use_native(cache):
        assert rows.dtype == cache.dtype and rows.stride(1) == 1 and rows.shape[1] == W
        native.check(
            native.kernels().hds_paged_rows(native.dt(cache), int(to_cache), cache.data_ptr(), rows.data_ptr(),
                                            rows.stride(0), seq.data_ptr(), pos.data_ptr(), native.ptr(dst_row),
                                            tables.data_ptr(), tables.shape[1], bs, W, n, native.stream()),
            "paged_rows")
        return
    p = pos.long()
    blk = tables[seq.long(), p // bs].long()
    dst = torch.arange(n) if dst_row is None else dst_row.long()
    if to_cache:
        cache[blk, p % bs] = rows[dst].to(cache.dtype)
    else:
        rows[dst] = cache[blk, p % bs].to(rows.dtype)


# -----------------------------------------------------------------------------------------------------------------
# heads with norms, convolutions, rotation, window, chunks, soft cap, sink, value mixing, output gate
# -----------------------------------------------------------------------------------------------------------------
@dataclass(frozen=True)
class HeadShape:
    heads: int
    kv_heads: int
    dim: int        # of a query / key head
    vdim: int       # of a value head
    window: int     # 0: every earlier token
    scale: float
    eps: float      # of the query / key norms
    gated: bool     # the projection ends with gate columns, one per query head
    gate_width: int = 1   # .. or, vdim: one per element of the heads' outputs
    chunk: int = 0        # positions see their own run of this many, counted from the sequence's start; 0: no chunks
    softcap: float = 0.0  # 0: none
    keep: int = 0         # of a window: the sequence's first positions, which stay visible
    # between projection and attention (``head_prep``): a short convolution of q and k, norms over all heads of q (of k),
    # rotation of the first ``rot`` dimensions of a head (neighbouring pairs); the keys as convolved may be the values
    prep: bool = False
    taps: int = 1
    rot: int = 0
    shared: bool = False

    @property
    def row(self):
        return self.kv_heads * (self.dim + self.vdim)

    @property
    def span(self):
        """The most keys a position sees; 0: no bound."""
        bounds = [b + self.keep for b in (self.window, self.chunk) if b]
        return min(bounds) if bounds else 0

    @property
    def channels(self):
        """q and k columns of the projection."""
        return (self.heads + self.kv_heads) * self.dim

    @property
    def qkv_width(self):
        return self.channels + (0 if self.shared else self.kv_heads * self.vdim)

    @property
    def state_floats(self):
        """The convolution's last inputs, a ring [taps, channels]: the input of position p is entry p % taps."""
        return self.taps * self.channels if self.taps > 1 else 0

    @property
    def width(self):
        return self.qkv_width + (self.heads * self.gate_width if self.gated else 0)


# Sequences with at most this many new tokens run token by token on the split-key kernel, the others in row blocks on
# the matrix cores
DECODE_MAX = 8


@dataclass
class HeadPlan:
    """Which tokens of a step run one by one, and the row blocks of the other sequences."""
    n_dec: int
    toks: Optional[torch.Tensor] = None   # None: every token, in order
    n_atoms: int = 0
    atoms: Optional[torch.Tensor] = None  # [n_atoms, 3] sequence, kv head, first row


def make_head_plan(seq_meta_host, n_tokens, heads, kv_heads, blocks, device, decode_max=None):
    """The plan of one batch for layers with these head counts; one host-to-device copy, shared by the layers.
    ``blocks`` False: every token runs one by one."""
    decode_max = DECODE_MAX if decode_max is None else decode_max
    if not blocks or all(n <= decode_max for (_, n, _) in seq_meta_host):
        return HeadPlan(n_tokens)
    toks, atoms, G = [], [], heads // kv_heads
    for s, (q0, n, _) in enumerate(seq_meta_host):
        if n <= decode_max:
            toks += range(q0, q0 + n)
            continue
        # the last rows of a portion see the most keys: start them first
        starts = range(0, n * G, ROWS_PER_ATOM)[::-1]
        atoms += [(s, hk, r0) for r0 in starts for hk in range(kv_heads)]
    flat = torch.tensor([v for a in atoms for v in a] + toks, dtype=torch.int32)
    if device.type == "cuda":
        flat = flat.pin_memory()
    dev = flat.to(device, non_blocking=True)
    k = 3 * len(atoms)
    plan = HeadPlan(len(toks), dev[k:], len(atoms), dev[:k].view(-1, 3))
    plan._keep = flat  # pinned source of an asynchronous copy
    return plan


def head_blocks_ok(shape, dtype):
    """Do the matrix-core and vector kernels take these heads (else the plain kernel)?"""
    return dtype == torch.bfloat16 and bool(native.kernels().hds_paged_attn_supported(shape.dim, shape.vdim))


def head_attention(qkv, shape, q_norm, k_norm, sink, cache, batch, plan, out, values=None, mix=None, gate=None,
                   prep=None):
    """qkv: [T, >= shape.width] projection, row by row q heads | k heads | v heads | gates (consumed); or with ``gate``
    [T, heads * gate_width] without the gates. q_norm / k_norm:
    [dim] float32 or None; sink: [heads] float32 or None; cache: [blocks, block_size, shape.row]. Appends the step's keys
    and values to ``cache`` and writes the gated heads into ``out`` [T, heads * vdim] (unit column stride). ``values``:
    [T, kv_heads * vdim] values of another layer, of which the share ``mix`` ([1] float32) goes into this layer's. ``prep`` (a HeadPrep, for shapes with
    ``prep``): q and k are convolved, normed and rotated first (q_norm, k_norm, values unused)."""
    sh, T = shape, qkv.shape[0]
    if sh.gated and gate is None:
        gate = qkv[:, sh.qkv_width:sh.width]
    assert sh.prep == (prep is not None)
    if prep is not None:
        from .head_prep import head_prep
        qkv = head_prep(qkv, sh, prep, cache, batch)
    if not native.use_native(qkv):
        return _head_attention_cpu(qkv, sh, q_norm, k_norm, sink, cache, batch, out, values, mix, gate)
    lib, st, dt = native.kernels(), native.stream(), native.dt(qkv)
    bs, tab = cache.shape[1], batch.block_tables
    mb = tab.shape[1]
    assert qkv.stride(1) == 1 and out.stride(1) == 1 and cache.dtype == qkv.dtype == out.dtype
    assert cache.shape[2] == sh.row and out.shape[1] == sh.heads * sh.vdim
    assert qkv.shape[1] >= (sh.heads * sh.dim if sh.prep else sh.qkv_width)
    if not sh.prep:
        native.check(
            lib.hds_head_norm_scatter(dt, qkv.data_ptr(), qkv.stride(0), native.ptr(q_norm), native.ptr(k_norm),
                                      cache.data_ptr(), batch.tok_seq.data_ptr(), batch.tok_pos.data_ptr(),
                                      tab.data_ptr(), T, mb, bs, sh.heads, sh.kv_heads, sh.dim, sh.vdim, float(sh.eps),
                                      native.ptr(values), 0 if values is None else values.stride(0),
                                      None if values is None else mix.data_ptr(), st), "head_norm_scatter")
    assert not sh.gated or (gate.shape == (T, sh.heads * sh.gate_width) and gate.stride(1) == 1 and gate.dtype == qkv.dtype)
    gp, ldg = (gate.data_ptr(), gate.stride(0)) if sh.gated else (None, 0)
    assert values is None or (values.shape == (T, sh.kv_heads * sh.vdim) and values.dtype == qkv.dtype)
    fast = head_blocks_ok(sh, qkv.dtype) and qkv.stride(0) % 8 == 0 and out.stride(0) % 8 == 0 and \
        qkv.data_ptr() % 16 == 0 and out.data_ptr() % 16 == 0 and (gp is None or sh.gate_width == 1 or
                                                                   (ldg % 4 == 0 and gp % 8 == 0))
    assert fast or not plan.n_atoms
    if plan.n_dec:
        n = plan.n_dec
        keys = min(mb * bs, sh.span) if sh.span else mb * bs
        splits = lib.hds_paged_decode_splits(n, sh.kv_heads if fast else sh.heads, keys)
        part_o = part_ml = None
        if splits > 1:
            part_o = torch.empty(n * sh.heads * splits * sh.vdim, device=qkv.device, dtype=torch.float32)
            part_ml = torch.empty(n * sh.heads * splits * 2, device=qkv.device, dtype=torch.float32)
        native.check(
            lib.hds_paged_decode(dt, int(not fast), qkv.data_ptr(), qkv.stride(0), cache.data_ptr(), out.data_ptr(),
                                 out.stride(0), native.ptr(part_o), native.ptr(part_ml), None, native.ptr(plan.toks),
                                 batch.tok_seq.data_ptr(), batch.tok_pos.data_ptr(), tab.data_ptr(), mb, bs, n,
                                 sh.heads, sh.kv_heads, sh.dim, sh.vdim, splits, float(sh.scale), sh.window,
                                 sh.chunk, sh.keep, float(sh.softcap), native.ptr(sink), gp, ldg, sh.gate_width,
                                 None, st), "paged_decode")
    if plan.n_atoms:
        native.check(
            lib.hds_paged_attn(qkv.data_ptr(), qkv.stride(0), cache.data_ptr(), out.data_ptr(), out.stride(0),
                               plan.atoms.data_ptr(), plan.n_atoms, batch.seq_meta.data_ptr(), tab.data_ptr(), mb, bs,
                               sh.heads, sh.kv_heads, sh.dim, sh.vdim, float(sh.scale), sh.window, sh.chunk, sh.keep,
                               float(sh.softcap), native.ptr(sink), gp, ldg, sh.gate_width, st),
            "paged_attn")
    return out


def _head_attention_cpu(qkv, sh, q_norm, k_norm, sink, cache, batch, out, values, mix, gate):
    T, H, G = qkv.shape[0], sh.heads, sh.kv_heads

    def normed(v, w):
        return v if w is None else v / torch.sqrt((v * v).mean(-1, keepdim=True) + sh.eps) * w

    if sh.prep:
        q = qkv.float().reshape(T, H, sh.dim)
    else:
        q, k, v = qkv[:, :sh.qkv_width].float().split([H * sh.dim, G * sh.dim, G * sh.vdim], 1)
        q = normed(q.reshape(T, H, sh.dim), q_norm)
        k = normed(k.reshape(T, G, sh.dim), k_norm).reshape(T, -1)
        if values is not None:
            v = (1 - mix) * v + mix * values.float()
        copy_rows(cache, torch.cat([k, v], 1), batch.tok_seq, batch.tok_pos, batch.block_tables, to_cache=True)
    gate = torch.sigmoid(gate.float()).reshape(T, H, sh.gate_width) if sh.gated else torch.ones(T, H, 1)
    bs = cache.shape[1]
    for s, (q0, n, seen) in enumerate(batch.seq_meta_host):
        if n == 0:
            continue
        lo = max(0, seen - sh.window + 1) if sh.window else 0
        if sh.chunk:
            lo = max(lo, seen - seen % sh.chunk)
        j = torch.cat([torch.arange(min(sh.keep, lo)), torch.arange(lo, seen + n)])
        rows = cache[batch.block_tables[s, j // bs].long(), j % bs].float()
        kk = rows[:, :G * sh.dim].view(-1, G, sh.dim).repeat_interleave(H // G, 1)
        vv = rows[:, G * sh.dim:].reshape(-1, G, sh.vdim).repeat_interleave(H // G, 1)
        sc = torch.einsum("thd,jhd->htj", q[q0:q0 + n], kk) * sh.scale
        if sh.softcap:
            sc = sh.softcap * torch.tanh(sc / sh.softcap)
        i = seen + torch.arange(n)
        hide = j[None] > i[:, None]
        if sh.window:
            hide |= (j[None] <= i[:, None] - sh.window) & (j[None] >= sh.keep)
        if sh.chunk:
            hide |= (j[None] < (i - i % sh.chunk)[:, None]) & (j[None] >= sh.keep)
        sc = sc.masked_fill(hide[None], float("-inf"))
        if sink is not None:
            sc = torch.cat([sc, sink.view(H, 1, 1).expand(H, n, 1)], -1)
        p = torch.softmax(sc, -1)[..., :j.numel()]
        o = torch.einsum("htj,jhd->thd", p, vv) * gate[q0:q0 + n]
        out[q0:q0 + n] = o.reshape(n, -1).to(out.dtype)
    return out
