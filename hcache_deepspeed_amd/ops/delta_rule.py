"""Gated delta rule over ragged batches (HIP, csrc/kernels/delta_rule.hip): short causal convolutions of q, k and v, unit
queries and keys, one decay and one step size per head, a 32-bit matrix state per head, gated RMS norm of the read-outs.

A sequence's state is one float32 row: S [heads, dim, vdim], then the convolution's last inputs as a ring [taps, channels]
(the input of position p is entry p % taps). A sequence without earlier tokens starts from zero. CPU tensors run the torch
implementation below."""
from dataclasses import dataclass
from typing import Optional

import torch

from . import native

UNIT_EPS = 1e-6

# Portions of a step are scanned by chunks on the matrix cores if one of them has more than this many tokens
SERIAL_MAX = 16


@dataclass(frozen=True)
class DeltaShape:
    heads: int
    kv_heads: int  # query and key heads, each shared by heads / kv_heads heads
    dim: int
    vdim: int
    taps: int
    eps: float     # of the read-outs' norm

    @property
    def channels(self):
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim

    @property
    def main_width(self):
        """Columns of the projection without b and a: q | k | v | output gate."""
        return self.channels + self.heads * self.vdim

    @property
    def width(self):
        return self.main_width + 2 * self.heads

    @property
    def state_floats(self):
        return self.heads * self.dim * self.vdim + self.taps * self.channels


@dataclass
class DeltaPlan:
    """Which sequences of a step run as single tokens and which as portions."""
    n_step: int
    step: Optional[torch.Tensor] = None  # None: all, in order
    n_scan: int = 0
    max_new: int = 0
    scan: Optional[torch.Tensor] = None


def step_ok(shape):
    return bool(native.kernels().hds_delta_step_ok(shape.dim, shape.vdim))


def make_delta_plan(seq_meta_host, n_seqs, max_new, single, device):
    """The plan of one batch; ``single``: lone tokens have a kernel of their own."""
    if max_new == 1 and single:
        return DeltaPlan(n_seqs)
    step = [s for s, (_, n, _) in enumerate(seq_meta_host) if n == 1] if single else []
    if not step:
        return DeltaPlan(0, n_scan=n_seqs, max_new=max_new)
    scan = [s for s, (_, n, _) in enumerate(seq_meta_host) if n > 1]
    host = torch.tensor(step + scan, dtype=torch.int32)
    if device.type == "cuda":
        host = host.pin_memory()
    dev = host.to(device, non_blocking=True)
    plan = DeltaPlan(len(step), dev[:len(step)], len(scan), max_new, dev[len(step):])
    plan._keep = host  # pinned source of an asynchronous copy
    return plan


def _chunk_floats(sh, dtype, n_tok, n_seqs):
    lib = native.kernels()
    per = lib.hds_delta_chunk_floats(native.dt(dtype), sh.dim, sh.vdim)
    return (n_tok // lib.hds_delta_chunk_tokens() + n_seqs) * sh.heads * per


def delta_rule(proj, shape, conv_w, a_log, dt_bias, norm_w, state, offset, batch, plan, out, ba=None):
    """proj: [T, >= shape.width], q | k | v | output gate | b | a; or with ``ba`` [T, >= 2 heads] (b | a) without these
    columns. conv_w: [taps, channels], the last row is the current token's; a_log, dt_bias: [heads];
    norm_w: [vdim], all float32. ``state[slot, offset:offset + shape.state_floats]`` is read and advanced; ``out``
    [T, heads * vdim] (unit column stride)."""
    if ba is None:
        assert proj.shape[1] >= shape.width
        ba = proj[:, shape.main_width:]
    if not native.use_native(proj):
        return _delta_rule_cpu(proj, ba, shape, conv_w, a_log, dt_bias, norm_w, state, offset, batch, out)
    sh, lib, dt, st = shape, native.kernels(), native.dt(proj), native.stream()
    T, dev = proj.shape[0], proj.device
    assert proj.stride(1) == 1 and out.stride(1) == 1 and out.dtype == proj.dtype and proj.shape[1] >= sh.main_width
    assert ba.dtype == proj.dtype and ba.shape[0] == T and ba.shape[1] >= 2 * sh.heads and ba.stride(1) == 1
    assert out.shape == (T, sh.heads * sh.vdim) and conv_w.shape == (sh.taps, sh.channels) and conv_w.is_contiguous()
    assert a_log.numel() == dt_bias.numel() == sh.heads and norm_w.numel() == sh.vdim
    assert offset + sh.state_floats <= state.shape[1]
    head = (dt, proj.data_ptr(), proj.stride(0), ba.data_ptr(), ba.stride(0), conv_w.data_ptr(), a_log.data_ptr(), dt_bias.data_ptr(),
            norm_w.data_ptr(), state.data_ptr() + 4 * offset, state.stride(0), batch.slots.data_ptr(),
            batch.seq_meta.data_ptr())
    dims = (sh.heads, sh.kv_heads, sh.dim, sh.vdim, sh.taps, float(sh.eps), st)
    if plan.n_step:
        native.check(lib.hds_delta_step(*head, native.ptr(plan.step), out.data_ptr(), out.stride(0), plan.n_step, *dims),
                     "delta_step")
    if plan.n_scan:
        f32 = dict(dtype=torch.float32, device=dev)
        y = torch.empty(T, sh.channels, dtype=proj.dtype, device=dev)
        rn, gb = torch.empty(T, 2 * sh.kv_heads, **f32), torch.empty(T, sh.heads, 2, **f32)
        aligned = all(t.stride(0) % 8 == 0 and t.data_ptr() % 16 == 0 for t in (proj, out))
        n_ws = _chunk_floats(sh, proj.dtype, T, plan.n_scan) if aligned and plan.max_new > SERIAL_MAX else 0
        ws = torch.empty(n_ws, **f32) if n_ws else None
        o = None if n_ws else torch.empty(T, sh.heads, sh.vdim, **f32)
        native.check(
            lib.hds_delta_scan(*head, native.ptr(plan.scan), y.data_ptr(), rn.data_ptr(), gb.data_ptr(), native.ptr(o),
                               native.ptr(ws), out.data_ptr(), out.stride(0), plan.n_scan, plan.max_new, *dims), "delta_scan")
    return out


def _silu(x):
    return x * torch.sigmoid(x)


def _delta_rule_cpu(proj, ba, sh, conv_w, a_log, dt_bias, norm_w, state, offset, batch, out):
    H, G, d, e, C, taps = sh.heads, sh.kv_heads, sh.dim, sh.vdim, sh.channels, sh.taps
    x, gate = proj[:, :sh.main_width].float().split([C, H * e], 1)
    b, a = ba[:, :2 * H].float().split(H, 1)
    decay = torch.exp(-torch.exp(a_log) * torch.nn.functional.softplus(a + dt_bias, threshold=40.0))
    beta = torch.sigmoid(b)
    n_state = H * d * e
    for s, (q0, n, seen) in enumerate(batch.seq_meta_host):
        row = state[batch.slots_host[s], offset:offset + sh.state_floats]
        S = row[:n_state].view(H, d, e)
        ring = row[n_state:].view(taps, C)
        cur = torch.zeros_like(S) if seen == 0 else S.clone()
        for t in range(n):
            pos = seen + t
            ring[pos % taps] = x[q0 + t]
            y = sum(conv_w[taps - 1 - k] * ring[(pos - k) % taps] for k in range(min(taps, pos + 1)))
            q, k, v = _silu(y).split([G * d, G * d, H * e])
            q, k = (u.view(G, d) / torch.sqrt((u.view(G, d)**2).sum(-1, keepdim=True) + UNIT_EPS) for u in (q, k))
            q, k = (u.repeat_interleave(H // G, 0) for u in (q * d**-0.5, k))
            cur = decay[q0 + t][:, None, None] * cur
            u = beta[q0 + t][:, None] * (v.view(H, e) - torch.einsum("hde,hd->he", cur, k))
            cur = cur + k[:, :, None] * u[:, None, :]
            o = torch.einsum("hde,hd->he", cur, q)
            o = o / torch.sqrt((o * o).mean(-1, keepdim=True) + sh.eps) * norm_w
            out[q0 + t] = (o.reshape(-1) * _silu(gate[q0 + t])).to(out.dtype)
        S.copy_(cur)
    return out
