"""Serving pre-norm over a 32-bit residual stream with a causal input convolution (HIP, csrc/kernels/input_norm.hip).

``input_norm`` adds the previous layer's output to the residual, RMS-norms the row once and writes, for each of up to
two sublayers k, ``h_k + conv_k(h_k)`` with ``h_k = g_k * norm(x)``; the last ``taps - 1`` normed rows of every
sequence live in its state slot. CPU tensors run the torch implementation below."""
import torch

from . import native
from .output_norm import norm_rows  # noqa: F401  (the norm at the other end of the stream)

MAX_TAPS = 16


def _rows_per_group(taps, max_new, n_tokens):
    if max_new == 1:
        return 1
    # rows plus history fill the workgroup's 8 waves once (short steps) or twice
    return max((8 if n_tokens <= 2048 else 16) - (taps - 1), taps - 1, 1)


def input_norm(x, delta, gains, convs, eps, taps, batch, state, offset, dtype, embed=None):
    """x: [T, W] float32 residual, or None: the rows of ``embed`` picked by ``batch.input_ids``. delta: [T, W] of
    ``dtype`` or None. gains: one or two float32 tensors ([1] or [W]); convs: as many [taps, W] float32 tensors or
    None. state: [slots, F] float32; the tail of a sequence is ``state[slot, offset:offset + (taps - 1) * W]``.
    Returns (new residual [T, W] float32, [y_k])."""
    T = batch.current_tokens
    W = x.shape[1] if x is not None else embed.shape[1]
    m = taps - 1
    ref = x if x is not None else embed
    x_out = torch.empty(T, W, dtype=torch.float32, device=ref.device)
    ys = [torch.empty(T, W, dtype=dtype, device=ref.device) for _ in gains]
    if native.use_native(ref):
        if taps > MAX_TAPS:
            raise NotImplementedError(f"input_norm: {taps} taps (at most {MAX_TAPS})")
        assert delta is None or (delta.dtype == dtype and delta.is_contiguous())
        two = len(gains) > 1
        sp = None if m == 0 else state.data_ptr() + 4 * offset
        g, w = list(gains), list(convs)
        native.check(
            native.kernels().hds_input_norm(
                native.dt(dtype), native.ptr(x), native.ptr(embed) if x is None else None,
                batch.input_ids.data_ptr() if x is None else None, native.ptr(delta), x_out.data_ptr(),
                g[0].data_ptr(), int(g[0].numel() > 1), native.ptr(w[0]), ys[0].data_ptr(),
                g[1].data_ptr() if two else None, int(two and g[1].numel() > 1), native.ptr(w[1]) if two else None,
                ys[1].data_ptr() if two else None, sp, 0 if m == 0 else state.stride(0), batch.slots.data_ptr(),
                batch.seq_meta.data_ptr(), batch.current_sequences, batch.max_new, W, taps,
                _rows_per_group(taps, batch.max_new, T), float(eps), native.stream()), "input_norm")
        return x_out, ys
    xs = embed[batch.input_ids].float() if x is None else x
    x_out.copy_(xs if delta is None else xs + delta.float())
    u = x_out / torch.sqrt((x_out * x_out).mean(-1, keepdim=True) + eps)
    for s, (q0, n, seen) in enumerate(batch.seq_meta_host):
        if n == 0:
            continue
        un = u[q0:q0 + n]
        if m:
            tail = state[batch.slots_host[s], offset:offset + m * W].view(m, W)
            old = torch.zeros_like(tail) if seen == 0 else tail.clone()
            full = torch.cat([old, un])
            tail.copy_(full[-m:])
        else:
            full = un
        for y, g, w in zip(ys, gains, convs):
            h = un.clone()
            if w is not None:
                for j in range(taps):
                    h += w[j] * full[j:j + n]
            y[q0:q0 + n] = (h * g).to(dtype)
    return x_out, ys
