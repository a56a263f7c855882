"""Norms on the output side of a sublayer over a 32-bit residual stream (HIP, csrc/kernels/output_norm.hip).

``residual_norm`` adds the normed output of a sublayer to the residual: ``x + g * norm(delta)``. The output may be a
plain matrix or an :class:`ops.experts.ExpertSum`, the parts of a routed expert layer's output, which the kernel sums on
the way in. It returns the new residual and the rows the next sublayer reads: rounded to the activations' type and
zero-padded to a multiple of ``pad`` columns (the 32-bit rows themselves where that changes nothing). ``embed_rows``
starts the stream, ``norm_rows`` is the output norm of selected rows. ``sandwich_norm`` is the step between two sublayers
with a norm on both sides: the residual sum of the first one's normed output and the second one's norm in one kernel.
``rms_rows`` norms column blocks, ``softcap_`` bounds logits. CPU tensors run the torch implementations."""
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
            p.y.data_ptr(), p.y.stride(0), p.expert.data_ptr(), p.weight.data_ptr(), native.ptr(p.row), native.ptr(sh),
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
