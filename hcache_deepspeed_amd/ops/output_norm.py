"""Norms on the output side of a sublayer over a 32-bit residual stream (HIP, csrc/kernels/output_norm.hip).

``residual_norm`` adds the normed output of a sublayer to the residual: ``x + g * norm(delta)``. The output may be a
plain matrix or an :class:`ops.experts.ExpertSum`, the parts of a routed expert layer's output, which the kernel sums on
the way in. It returns the new residual and the rows the next sublayer reads: rounded to the activations' type and
zero-padded to a multiple of ``pad`` columns (the 32-bit rows themselves where that changes nothing). ``embed_rows``
and ``embed_pairs`` start the stream, ``norm_rows`` is the output norm of selected rows. ``sandwich_norm`` is the step between two sublayers
with a norm on both sides: the residual sum of the first one's normed output and the second one's norm in one kernel;
``stream_norm`` is its general form (layer norms, a :class:`PairSum` or an ExpertSum as the output, no second norm, padded rows).
``rms_rows`` norms column blocks, ``softcap_`` bounds logits. CPU tensors run the torch implementations."""
from dataclasses import dataclass

import torch

from . import native


def padded(n, pad):
    return -(-n // pad) * pad


def _rounded(x, dtype, pad):
    """(tensor for the rounded rows, its row length); None where the 32-bit rows serve."""
    T, W = x.shape
    ld = padded(W, pad)
    if dtype == torch.float32 and ld == W:
        return None, W
    return torch.empty(T, ld, dtype=dtype, device=x.device), ld


def _fill(xb, x):
    if xb is None:
        return x
    xb[:, :x.shape[1]] = x.to(xb.dtype)
    xb[:, x.shape[1]:] = 0
    return xb


def embed_rows(embed, ids, scale, dtype, pad=1):
    """scale * embed[ids] in float32, and rounded."""
    n, W = ids.numel(), embed.shape[1]
    x = torch.empty(n, W, dtype=torch.float32, device=embed.device)
    xb, ld = _rounded(x, dtype, pad)
    if native.use_native(embed):
        assert embed.dtype == dtype and ids.dtype == torch.int64
        native.check(
            native.kernels().hds_embed_rows(native.dt(embed), embed.data_ptr(), ids.data_ptr(), float(scale),
                                            x.data_ptr(), native.ptr(xb), ld, n, W, embed.shape[0], native.stream()),
            "embed_rows")
        return x, x if xb is None else xb
    x.copy_(embed[ids].float() * scale)
    return x, _fill(xb, x)


def residual_norm(x, delta, gain, eps, dtype, pad=1):
    """x: [T, W] float32, updated in place; delta: [T, W] of ``dtype`` or an ExpertSum; gain: [W] float32."""
    T, W = x.shape
    xb, ld = _rounded(x, dtype, pad)
    plain = torch.is_tensor(delta)
    if native.use_native(x):
        assert gain.numel() == W and x.is_contiguous()
        lib = native.kernels()
        if plain:
            assert delta.dtype == dtype and delta.stride(1) == 1
            native.check(
                lib.hds_residual_norm(native.dt(dtype), x.data_ptr(), x.data_ptr(), native.ptr(xb), ld,
                                      delta.data_ptr(), delta.stride(0), gain.data_ptr(), T, W, float(eps),
                                      native.stream()), "residual_norm")
        else:
            _experts_norm(x, xb, ld, gain, None, delta, eps)
        return x, x if xb is None else xb
    d = delta.float() if plain else delta.total(x)
    x += d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * gain
    return x, _fill(xb, x)


def sum_experts(x, parts, dtype):
    """The sum of an ExpertSum as a [T, W] matrix of ``dtype`` (x: the residual, which identity choices return)."""
    out = torch.empty(x.shape, dtype=dtype, device=x.device)
    if native.use_native(x):
        _experts_norm(x, None, 0, None, out, parts, 0.0)
        return out
    return out.copy_(parts.total(x))


def _experts_norm(x, xb, ld, gain, out, p, eps):
    T, W = x.shape
    sh = p.shared
    native.check(
        native.kernels().hds_experts_norm(
            native.dt(p.y), x.data_ptr(), x.data_ptr(), native.ptr(xb), ld, native.ptr(gain), native.ptr(out),
            p.y.data_ptr(), p.y.stride(0), p.expert.data_ptr(), native.ptr(p.weight), native.ptr(p.row), native.ptr(sh),
            0 if sh is None else sh.stride(0), None if sh is None else p.gate.data_ptr(),
            0 if sh is None else p.gate.stride(0), p.n_experts, p.expert.shape[1], int(p.identity), T, W, float(eps),
            native.stream()), "experts_norm")


def norm_rows(x, delta, idx, gain, eps, dtype=None):
    """g * norm(x[idx] + delta[idx]) in delta's dtype (or ``dtype``; delta may be None): [len(idx), W]. idx: int32."""
    W = x.shape[1]
    y = torch.empty(idx.numel(), W, dtype=dtype or delta.dtype, device=x.device)
    if native.use_native(x):
        assert delta is None or delta.dtype == y.dtype
        native.check(
            native.kernels().hds_norm_rows(native.dt(y), x.data_ptr(), native.ptr(delta), idx.data_ptr(),
                                           gain.data_ptr(), int(gain.numel() > 1), y.data_ptr(), idx.numel(), W,
                                           float(eps), native.stream()), "norm_rows")
        return y
    h = x[idx.long()]
    if delta is not None:
        h = h + delta[idx.long()].float()
    y.copy_(h / torch.sqrt((h * h).mean(-1, keepdim=True) + eps) * gain)
    return y


def _rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


@dataclass
class PairSum:
    """(ga * rms(a) + gb * rms(b)) / 2: two outputs of one sublayer, each normed by itself. a, b: [T, W]; gains: [W] float32."""
    a: torch.Tensor
    b: torch.Tensor
    ga: torch.Tensor
    gb: torch.Tensor

    def total(self, eps):
        return 0.5 * (self.ga * _rms(self.a.float(), eps) + self.gb * _rms(self.b.float(), eps))


def _normed(x, norm, eps):
    """norm: an RMS norm's gain, or (gain, bias) of a layer norm."""
    if torch.is_tensor(norm):
        return norm * _rms(x, eps)
    d = x - x.mean(-1, keepdim=True)
    return norm[0] * _rms(d, eps) + norm[1]


def stream_norm(x, delta, norm, next_norm, eps, dtype, idx=None, pad=1):
    """(x' = x + norm(delta), next_norm(x') in ``dtype``, zero-padded to a multiple of ``pad`` columns). x: [T, W] float32,
    updated in place; delta: [T, W] of ``dtype``, a PairSum, an ExpertSum or None (x' = x). A norm is the gain [W] of an
    RMS norm or (gain, bias) of a layer norm, float32; next_norm None: the rows of x' themselves. ``idx`` (int32): only these
    rows, and the first result is None."""
    W = x.shape[1]
    n = x.shape[0] if idx is None else idx.numel()
    ld = padded(W, pad)
    same = next_norm is None and idx is None and dtype == torch.float32 and ld == W  # x' serves as the rows
    y = None if same else torch.empty(n, ld, dtype=dtype, device=x.device)
    pair = isinstance(delta, PairSum)
    plain = delta is None or torch.is_tensor(delta)
    if native.use_native(x):
        if same and delta is None:
            return x, x
        assert x.is_contiguous() and x.dtype == torch.float32

        def split(m):
            w, b = (m, None) if m is None or torch.is_tensor(m) else m
            assert all(v is None or (v.numel() == W and v.dtype == torch.float32) for v in (w, b))
            return native.ptr(w), native.ptr(b)

        first, other = (delta.a, delta.b) if pair else (delta if plain else None, None)
        for v in (first, other):
            assert v is None or (v.dtype == dtype and v.stride(1) == 1 and v.shape[1] == W and v.shape[0] == x.shape[0])
        parts = [None, 0] + [None] * 4 + [0, None, 0, 0, 0, 0]
        if not (plain or pair):
            sh = delta.shared
            assert delta.y.dtype == dtype and delta.expert.shape[0] == x.shape[0]
            parts = [delta.y.data_ptr(), delta.y.stride(0), delta.expert.data_ptr(), native.ptr(delta.weight),
                     native.ptr(delta.row), native.ptr(sh), 0 if sh is None else sh.stride(0),
                     None if sh is None else delta.gate.data_ptr(), 0 if sh is None else delta.gate.stride(0),
                     delta.n_experts, delta.expert.shape[1], int(delta.identity)]
        native.check(
            native.kernels().hds_stream_norm(
                native.dt(dtype), 0 if plain else (1 if pair else 2), x.data_ptr(), native.ptr(first),
                0 if first is None else first.stride(0), native.ptr(other), 0 if other is None else other.stride(0),
                native.ptr(delta.ga if pair else None), native.ptr(delta.gb if pair else None), *parts, *split(norm),
                *split(next_norm), native.ptr(idx), None if idx is not None or delta is None else x.data_ptr(),
                native.ptr(y), ld, n, W, float(eps), native.stream()), "stream_norm")
        return None if idx is not None else x, x if same else y
    d = delta
    if not plain:
        d = delta.total(eps) if pair else delta.total(x)
    h = x if idx is None else x[idx.long()]
    if d is not None:
        h = h + _normed((d if idx is None else d[idx.long()]).float(), norm, eps)
    if idx is None:
        x.copy_(h)
    if same:
        return x, x
    return None if idx is not None else x, _fill(y, h if next_norm is None else _normed(h, next_norm, eps))


def embed_pairs(embed, pairs, ids, scale, mul_prev, mul_cur, state, offset, batch):
    """scale * embed[ids] + pairs[(previous id * mul_prev + id * mul_cur) mod buckets] in float32; pairs: [buckets + 1, W], its
    last row for a sequence's first token. ``state[slot, offset]`` keeps a sequence's last token (as an int32)."""
    n, W = ids.numel(), embed.shape[1]
    buckets = pairs.shape[0] - 1
    if native.use_native(embed):
        x = torch.empty(n, W, dtype=torch.float32, device=embed.device)
        assert embed.dtype == pairs.dtype and ids.dtype == torch.int64 and embed.is_contiguous() and pairs.is_contiguous()
        native.check(
            native.kernels().hds_embed_pairs(native.dt(embed), embed.data_ptr(), pairs.data_ptr(), ids.data_ptr(),
                                             float(scale), batch.tok_seq.data_ptr(), batch.seq_meta.data_ptr(),
                                             batch.slots.data_ptr(), state.data_ptr() + 4 * offset, state.stride(0),
                                             x.data_ptr(), n, W, embed.shape[0], buckets, mul_prev, mul_cur,
                                             native.stream()), "embed_pairs")
        return x
    at = torch.empty_like(ids)
    last = state.view(torch.int32)[:, offset]
    for s, (q0, k, seen) in enumerate(batch.seq_meta_host):
        slot = batch.slots_host[s]
        before = torch.cat([last[slot:slot + 1].long(), ids[q0:q0 + k - 1]])
        at[q0:q0 + k] = (before * mul_prev + ids[q0:q0 + k] * mul_cur) % buckets
        if seen == 0:
            at[q0] = buckets
        last[slot] = ids[q0 + k - 1].to(torch.int32)
    return embed[ids].float() * scale + pairs[at].float()


def sandwich_norm(x, delta, gain, next_gain, eps, dtype, embed=None, idx=None):
    """(x' = x + gain * norm(delta), next_gain * norm(x') in ``dtype``). x: [T, W] float32, updated in place; or None, then
    ``embed`` = (table, ids, scale) starts the stream. delta: [T, W] of ``dtype`` or None (x' = x). gains: [W] float32.
    ``idx`` (int32): only these rows, and the first result is None."""
    table, ids, scale = embed if x is None else (None, None, 1.0)
    W = table.shape[1] if x is None else x.shape[1]
    n = idx.numel() if idx is not None else (ids.numel() if x is None else x.shape[0])
    dev = table.device if x is None else x.device
    out = None if idx is not None else (x if x is not None else torch.empty(n, W, dtype=torch.float32, device=dev))
    y = torch.empty(n, W, dtype=dtype, device=dev)
    if native.use_native(y):
        assert delta is None or (delta.dtype == dtype and delta.stride(1) == 1 and gain.numel() == W)
        assert next_gain.numel() == W and (x is None or x.is_contiguous()) and (table is None or table.dtype == dtype)
        native.check(
            native.kernels().hds_sandwich_norm(
                native.dt(dtype), native.ptr(x), native.ptr(table), native.ptr(ids), float(scale), native.ptr(delta),
                0 if delta is None else delta.stride(0), native.ptr(gain), next_gain.data_ptr(), native.ptr(idx),
                native.ptr(out), y.data_ptr(), n, W, 0 if table is None else table.shape[0], float(eps),
                native.stream()), "sandwich_norm")
        return out, y
    h = table[ids].float() * scale if x is None else x
    if idx is not None:
        h, delta = h[idx.long()], None if delta is None else delta[idx.long()]
    if delta is not None:
        h = h + gain * _rms(delta.float(), eps)
    if out is not None:
        out.copy_(h)
    return out, y.copy_(next_gain * _rms(h, eps))


def rms_rows(x, gain, eps):
    """gain * norm(x) of rows [T, W] (any row stride), contiguous."""
    y = torch.empty(x.shape, dtype=x.dtype, device=x.device)
    if native.use_native(x):
        assert x.stride(1) == 1 and gain.numel() == x.shape[1]
        native.check(
            native.kernels().hds_row_norm(native.dt(x), x.data_ptr(), x.stride(0), gain.data_ptr(), y.data_ptr(),
                                          y.stride(0), x.shape[0], x.shape[1], float(eps), native.stream()), "row_norm")
        return y
    return y.copy_(gain * _rms(x.float(), eps))


def softcap_(x, cap):
    """cap * tanh(x / cap) in place (contiguous)."""
    if native.use_native(x):
        assert x.is_contiguous()
        native.check(native.kernels().hds_softcap(native.dt(x), x.data_ptr(), x.numel(), float(cap), native.stream()),
                     "softcap")
        return x
    return x.copy_(cap * torch.tanh(x.float() / cap))
