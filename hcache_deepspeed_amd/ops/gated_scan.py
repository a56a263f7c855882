"""Gated linear recurrence of the minGRU mixer over ragged batches (HIP, csrc/kernels/gated_scan.hip; the decode step
fused with its projection: csrc/kernels/gemv.hip). States are float32 rows of the sequences' slots; a sequence without
earlier tokens starts from zero. CPU tensors run the torch implementation below."""
import torch

from . import native


def gated_scan(proj, bias_z, bias_x, out, batch, state, offset):
    """proj: [T, 3 W] (update gate | candidate | output gate); out: [T, W] view with unit column stride;
    ``state[slot, offset:offset + W]`` is read and advanced."""
    W = out.shape[1]
    if native.use_native(proj):
        assert proj.stride(1) == 1 and out.stride(1) == 1 and out.dtype == proj.dtype
        native.check(
            native.kernels().hds_gated_scan(native.dt(proj), proj.data_ptr(), proj.stride(0), bias_z.data_ptr(),
                                            bias_x.data_ptr(), out.data_ptr(), out.stride(0),
                                            state.data_ptr() + 4 * offset, state.stride(0), batch.slots.data_ptr(),
                                            batch.seq_meta.data_ptr(), batch.current_sequences, batch.max_new, W,
                                            native.stream()), "gated_scan")
        return out
    a, b, g = proj.float().split(W, 1)
    a, b = a + bias_z, b + bias_x
    keep, add = torch.sigmoid(-a), torch.sigmoid(a) * torch.where(b >= 0, b + 0.5, torch.sigmoid(b))
    for s, (q0, n, seen) in enumerate(batch.seq_meta_host):
        st = state[batch.slots_host[s], offset:offset + W]
        cur = torch.zeros_like(st) if seen == 0 else st.clone()
        for t in range(q0, q0 + n):
            cur = keep[t] * cur + add[t]
            out[t] = (cur * g[t] * torch.sigmoid(g[t])).to(out.dtype)
        st.copy_(cur)
    return out


def recur_step_ok(x, w, max_rows=8):
    """Can ``recur_step`` take these rows (bf16, one new token per sequence, 16-B rows)?"""
    return (native.use_native(x) and x.dtype == torch.bfloat16 and torch.is_tensor(w) and w.dtype == torch.bfloat16
            and 1 <= x.shape[0] <= max_rows and x.shape[1] % 8 == 0 and x.stride(1) == 1 and x.stride(0) % 8 == 0
            and w.is_contiguous() and x.data_ptr() % 16 == 0 and w.data_ptr() % 16 == 0)


def recur_step(x, w, bias_z, bias_x, out, batch, state, offset):
    """Projection and recurrence of a decode step in one kernel: row m of x is sequence m's one new token."""
    M, K = x.shape
    W = out.shape[1]
    assert w.shape == (3 * W, K) and M == batch.current_sequences
    native.check(
        native.kernels().hds_gemv_recur_bf16(x.data_ptr(), w.data_ptr(), bias_z.data_ptr(), bias_x.data_ptr(),
                                             out.data_ptr(), state.data_ptr() + 4 * offset, state.stride(0),
                                             batch.slots.data_ptr(), batch.seq_meta.data_ptr(), M, W, K, x.stride(0),
                                             out.stride(0), native.stream()), "gemv_recur")
    return out
