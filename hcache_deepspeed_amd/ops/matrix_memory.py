"""Matrix memories over ragged batches (HIP, csrc/kernels/matrix_memory.hip): linear attention with a decay per head and a
32-bit state, its read-outs normed per head and gated. Two kinds: a fixed decay (retention), and exponential input and
forget gates under a running maximum with a normalizer (the mLSTM of xLSTM).

A sequence's state is one float32 row: per head S [dim, vdim], with the gated kind followed by the normalizer n [dim] (and
padded to a multiple of 4), then behind all heads of the gated kind the running maxima [heads]. A sequence without earlier
tokens starts from zero. CPU tensors run the torch implementation below."""
from dataclasses import dataclass

import torch

from . import native
from .delta_rule import make_delta_plan

FLOOR_EPS = 1e-6

# Portions of a step are scanned by chunks on the matrix cores if one of them has more than this many tokens
SERIAL_MAX = 16

GATES = {"sigmoid": 0, "silu": 1}

make_memory_plan = make_delta_plan  # lone tokens and portions, as for the delta rule


@dataclass(frozen=True)
class MemoryShape:
    heads: int
    dim: int
    vdim: int
    eps: float          # of the read-outs' norm
    gate: str           # of the outputs: sigmoid | silu
    gated: bool         # exponential input and forget gates (else a fixed decay per head)
    cap: float = 0.0    # of the gates' logits
    rot: int = 0        # rotated dimensions of q and k (neighbouring pairs)

    @property
    def main_width(self):
        """Columns of the projection without the gates of the recurrence: q | k | v | output gate."""
        return 2 * self.heads * (self.dim + self.vdim)

    @property
    def width(self):
        return self.main_width + (2 * self.heads if self.gated else 0)

    @property
    def head_floats(self):
        return -(-(self.dim * self.vdim + (self.dim if self.gated else 0)) // 4) * 4

    @property
    def state_floats(self):
        return self.heads * self.head_floats + (self.heads if self.gated else 0)


def step_ok(shape):
    return bool(native.kernels().hds_memory_step_ok(shape.dim, shape.vdim))


def _chunk_floats(sh, dtype, n_tok, n_seqs):
    lib = native.kernels()
    per = lib.hds_memory_chunk_floats(native.dt(dtype), sh.dim, sh.vdim, int(sh.gated))
    return (n_tok // lib.hds_memory_chunk_tokens() + n_seqs) * sh.heads * per


def matrix_memory(proj, shape, w, tables, state, offset, batch, plan, out):
    """proj: [T, >= shape.width], q | k | v | output gate and, of the gated kind, input | forget gate. w: float32 tensors,
    "log_decay" [heads], or "i.b" and "f.b" [heads]; "norm" [heads * vdim] or None. tables: (cos, sin) [positions, rot / 2] or
    None. ``state[slot, offset:offset + shape.state_floats]`` is read and advanced; ``out`` [T, heads * vdim] (unit column
    stride)."""
    sh, T = shape, proj.shape[0]
    assert proj.shape[1] >= sh.width and out.shape == (T, sh.heads * sh.vdim) and offset + sh.state_floats <= state.shape[1]
    norm = w["norm"]
    assert norm is None or norm.numel() == sh.heads * sh.vdim
    assert all(w[k].numel() == sh.heads for k in (("i.b", "f.b") if sh.gated else ("log_decay", )))
    if not native.use_native(proj):
        return _matrix_memory_cpu(proj, sh, w, tables, state, offset, batch, out)
    lib, dt, st, dev = native.kernels(), native.dt(proj), native.stream(), proj.device
    assert proj.stride(1) == 1 and out.stride(1) == 1 and out.dtype == proj.dtype and offset % 4 == 0
    cos, sin = tables if sh.rot else (None, None)
    assert not sh.rot or cos.shape[1] == sh.rot // 2
    decay, bi, bf = (None, w["i.b"], w["f.b"]) if sh.gated else (w["log_decay"], None, None)

    def run(single, seqs, n_seqs, max_new, coef, o, chunks):
        native.check(
            lib.hds_memory(dt, single, proj.data_ptr(), proj.stride(0), native.ptr(decay), native.ptr(bi), native.ptr(bf),
                           float(sh.cap), native.ptr(cos), native.ptr(sin), sh.rot, native.ptr(norm), GATES[sh.gate],
                           state.data_ptr() + 4 * offset, state.stride(0), batch.slots.data_ptr(),
                           batch.seq_meta.data_ptr(), native.ptr(seqs), native.ptr(coef), native.ptr(o),
                           native.ptr(chunks), out.data_ptr(), out.stride(0), n_seqs, max_new, sh.heads, sh.dim, sh.vdim,
                           float(sh.eps), st), "matrix_memory")

    if plan.n_step:
        run(1, plan.step, plan.n_step, 1, None, None, None)
    if plan.n_scan:
        aligned = all(t.stride(0) % 8 == 0 and t.data_ptr() % 16 == 0 for t in (proj, out)) and state.stride(0) % 4 == 0
        n_ws = _chunk_floats(sh, proj.dtype, T, plan.n_scan) if aligned and plan.max_new > SERIAL_MAX else 0
        f32 = dict(dtype=torch.float32, device=dev)
        if n_ws:
            run(0, plan.scan, plan.n_scan, plan.max_new, None, None, torch.empty(n_ws, **f32))
        else:
            coef = torch.empty(T, sh.heads, 4, **f32) if sh.gated else None
            run(0, plan.scan, plan.n_scan, plan.max_new, coef, torch.empty(T, sh.heads, sh.vdim, **f32), None)
    return out


def rotate_pairs(x, cos, sin):
    """x [..., heads, dim]: the neighbouring pairs of its first 2 * cos.shape[-1] dimensions turned; cos, sin [..., pairs]."""
    n = 2 * cos.shape[-1]
    a, b = x[..., 0:n:2], x[..., 1:n:2]
    c, s = cos.unsqueeze(-2), sin.unsqueeze(-2)
    return torch.cat([torch.stack([a * c - b * s, b * c + a * s], -1).flatten(-2), x[..., n:]], -1)


def _matrix_memory_cpu(proj, sh, w, tables, state, offset, batch, out):
    H, d, e = sh.heads, sh.dim, sh.vdim
    T = proj.shape[0]
    q, k, v, gate = proj[:, :sh.main_width].float().split([H * d, H * d, H * e, H * e], 1)
    q, k, v = q.reshape(T, H, d), k.reshape(T, H, d), v.reshape(T, H, e)
    if sh.rot:
        pos = batch.tok_pos.long()
        q, k = (rotate_pairs(x, tables[0][pos], tables[1][pos]) for x in (q, k))
    q = q * d**-0.5
    if sh.gated:
        zi, zf = proj[:, sh.main_width:sh.width].float().split(H, 1)
        i = sh.cap * torch.tanh((zi + w["i.b"]) / sh.cap)
        f = torch.nn.functional.logsigmoid(sh.cap * torch.tanh((zf + w["f.b"]) / sh.cap))
    else:
        i, f = torch.zeros(T, H), w["log_decay"].expand(T, H)
    gate = torch.sigmoid(gate) * (gate if sh.gate == "silu" else 1.0)
    for s, (q0, n, seen) in enumerate(batch.seq_meta_host):
        row = state[batch.slots_host[s], offset:offset + sh.state_floats]
        heads = row[:H * sh.head_floats].view(H, sh.head_floats)
        S, norm = heads[:, :d * e].reshape(H, d, e).clone(), heads[:, d * e:d * e + d].clone()
        m = row[H * sh.head_floats:].clone() if sh.gated else torch.zeros(H)
        if seen == 0:
            S, norm, m = torch.zeros_like(S), torch.zeros_like(norm), torch.zeros_like(m)
        for t in range(q0, q0 + n):
            now = torch.maximum(f[t] + m, i[t])
            keep, add = torch.exp(f[t] + m - now), torch.exp(i[t] - now)
            m = now
            S = keep[:, None, None] * S + (add[:, None] * k[t])[:, :, None] * v[t][:, None, :]
            o = torch.einsum("hde,hd->he", S, q[t])
            if sh.gated:
                norm = keep[:, None] * norm + add[:, None] * k[t]
                o = o / (torch.maximum((norm * q[t]).sum(-1).abs(), torch.exp(-m)) + FLOOR_EPS)[:, None]
            o = (o / torch.sqrt((o * o).mean(-1, keepdim=True) + sh.eps)).reshape(-1)
            out[t] = (o * (1.0 if w["norm"] is None else w["norm"]) * gate[t]).to(out.dtype)
        heads[:, :d * e] = S.reshape(H, -1)
        if sh.gated:
            heads[:, d * e:d * e + d] = norm
            row[H * sh.head_floats:] = m
    return out
