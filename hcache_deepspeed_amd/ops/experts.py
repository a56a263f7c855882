"""Routed expert layer of the serving engine (HIP, csrc/kernels/experts.hip and grouped_gemm.hip).

The router scores experts and *identity* experts (which return their input and have no weights) by a softmax or by
sigmoids; a correction may decide, without weighing, which are chosen, and only the best groups of neighbours take part. A
choice's weight multiplies the expert's output, or its input. An optional shared expert sees every token through a sigmoid
gate. ``routed_experts`` returns the layer's output in parts
(:class:`ExpertSum`); ops/output_norm.py sums them where the sum is used. CPU tensors run the torch implementation."""
from dataclasses import dataclass
from typing import Optional

import torch
import torch.nn.functional as F

from . import native
from .activations import glu_rows

PAD = 128  # bf16 expert weights: every dimension is zero-padded to a multiple of the grouped product's tile

# Steps of at most this many tokens run the experts straight from the choices; longer ones sort them by expert first
SKINNY_TOKENS = 64


@dataclass(frozen=True)
class RouterShape:
    experts: int
    identity: int = 0
    top: int = 1
    groups: int = 1
    keep: int = 1
    scale: float = 1.0
    score: str = "softmax"     # or "sigmoid"
    weigh_input: bool = False  # the weights multiply what the experts read instead of what they return

    @property
    def outputs(self):
        return self.experts + self.identity

    def check(self):
        n = self.outputs
        if self.score not in ("softmax", "sigmoid") or (self.weigh_input and self.identity):
            raise NotImplementedError(f"router {self}: scores {self.score!r}, weighed inputs with identity experts")
        if n > 1024 or self.groups > 64 or n % self.groups or not 1 <= self.keep <= self.groups or \
                not 1 <= self.top <= self.keep * (n // self.groups):
            raise NotImplementedError(f"router {self}: at most 1024 outputs in at most 64 equal groups, "
                                      "top of them inside the kept groups")


@dataclass
class ExpertSum:
    """sum_j weight[t, j] * (y[row[t, j]] or the input) + sigmoid(gate[t]) * shared[t]."""
    y: torch.Tensor                # [rows, >= W]
    expert: torch.Tensor           # [T, k] int32; n_experts and above: identity
    weight: Optional[torch.Tensor]  # [T, k] float32; None: ones
    row: Optional[torch.Tensor]    # [T, k] int32; None: rows in order of the choices
    n_experts: int
    shared: Optional[torch.Tensor] = None  # [T, >= W]
    gate: Optional[torch.Tensor] = None    # [T] float32, any stride
    identity: bool = True          # False: another rank of the tensor-parallel group adds the identity experts

    def total(self, x):
        T, W = x.shape
        row = torch.arange(self.expert.numel()).view_as(self.expert) if self.row is None else self.row.long()
        own = self.expert < self.n_experts
        y = self.y[torch.where(own, row, 0)][..., :W].float()
        y = torch.where(own[..., None], y, x[:, None] if self.identity else torch.zeros(()))
        out = (y if self.weight is None else y * self.weight[..., None]).sum(1)
        if self.shared is not None:
            out = out + torch.sigmoid(self.gate)[:, None] * self.shared[:, :W].float()
        return out


def route(z, correction, shape):
    """correction: [outputs] float32 or None; z: [T, >= outputs] float32 router logits -> (expert [T, top] int32, weight [T, top] float32)."""
    T, n = z.shape[0], shape.outputs
    if native.use_native(z):
        expert = torch.empty(T, shape.top, dtype=torch.int32, device=z.device)
        weight = torch.empty(T, shape.top, dtype=torch.float32, device=z.device)
        assert z.dtype == torch.float32 and z.stride(1) == 1
        assert correction is None or (correction.dtype == torch.float32 and correction.numel() == n)
        native.check(
            native.kernels().hds_router_select(z.data_ptr(), z.stride(0), int(shape.score == "sigmoid"),
                                               native.ptr(correction), expert.data_ptr(), weight.data_ptr(), T, n, shape.groups, shape.keep, shape.top,
                                               float(shape.scale), native.stream()), "router_select")
        return expert, weight
    s = torch.sigmoid(z[:, :n]) if shape.score == "sigmoid" else torch.softmax(z[:, :n], -1)
    c = s if correction is None else s + correction
    if shape.keep < shape.groups:
        by_group = c.view(T, shape.groups, -1)
        best = by_group.amax(-1).topk(shape.keep, -1).indices
        drop = torch.ones(T, shape.groups, dtype=torch.bool).scatter_(1, best, False)
        c = by_group.masked_fill(drop[..., None], float("-inf")).view(T, n)
    expert = c.topk(shape.top, -1).indices
    return expert.to(torch.int32), s.gather(1, expert) * shape.scale


def _shared_product(x, w):
    """Gate / up product, activation and down product of the shared expert for a long step."""
    gu = F.linear(x, w["ws13"])
    h = torch.empty(x.shape[0], w["ws2"].shape[1], dtype=x.dtype, device=x.device)
    return F.linear(glu_rows(gu, "silu", h), w["ws2"])


def routed_experts(x, w, shape, identity=True, act="silu", limit=0.0):
    """act: "silu", or the "clamped" unit with ``limit``. x: [T, K] rows (bf16: zero-padded to K, a multiple of PAD; float32: the residual itself). w: "router.w"
    [outputs (+ 1: the shared expert's gate), K], "router.c" [outputs] float32 or None, "w13" [E, 2 I, K] (gate rows, then up
    rows), "w2" [E, W, I], and "ws13", "ws2" of the shared expert or None."""
    T, K = x.shape
    k, E = shape.top, shape.experts
    w13, w2, ws13, ws2 = w["w13"], w["w2"], w["ws13"], w["ws2"]
    inter, out_w, has_shared = w2.shape[2], w2.shape[1], w["ws13"] is not None
    R = shape.outputs + int(has_shared)
    assert w["router.w"].shape == (R, K) and w13.shape == (E, 2 * inter, K)
    if not native.use_native(x):
        return _routed_experts_cpu(x, w, shape, identity, act, limit)
    code, limit = {"silu": 0, "clamped": 5}[act], float(limit)
    assert not has_shared or act == "silu"
    lib, st, dev = native.kernels(), native.stream(), x.device
    fast = x.dtype == torch.bfloat16
    assert x.stride(1) == 1 and all(t is None or (t.dtype == x.dtype and t.is_contiguous())
                                    for t in (w["router.w"], w13, w2, ws13, ws2))
    if fast:
        z = torch.empty(T, R, dtype=torch.float32, device=dev)
        native.check(lib.hds_router_logits(x.data_ptr(), x.stride(0), w["router.w"].data_ptr(), z.data_ptr(), R, T, R,
                                           K, st), "router_logits")
    else:
        z = F.linear(x, w["router.w"])
    expert, weight = route(z, w["router.c"], shape)
    weigh_in = weight if shape.weigh_input else None
    parts = ExpertSum(None, expert, None if shape.weigh_input else weight, None, E, identity=identity)
    if has_shared:
        parts.gate = z[:, shape.outputs]
    n = T * k
    if fast and T <= SKINNY_TOKENS and n <= lib.hds_experts_skinny_max():
        h = torch.empty(n, inter, dtype=x.dtype, device=dev)
        parts.y = torch.empty(n, out_w, dtype=x.dtype, device=dev)
        hs, si = None, 0
        if has_shared:
            si = ws2.shape[1]
            hs = torch.empty(T, si, dtype=x.dtype, device=dev)
            parts.shared = torch.empty(T, out_w, dtype=x.dtype, device=dev)
        for glu, src, ld, kx, wt, dst, N, kk, ss, ws, sd, Ns, Ks in (
                (1, x, x.stride(0), k, w13, h, inter, K, x, ws13, hs, si, K),
                (0, h, inter, 1, w2, parts.y, out_w, inter, hs, ws2, parts.shared, out_w, si)):
            native.check(
                lib.hds_experts_skinny(glu, src.data_ptr(), ld, wt.data_ptr(), dst.data_ptr(), N, expert.data_ptr(), n,
                                       kx, E, N, kk, native.ptr(ss), 0 if ss is None else ss.stride(0),
                                       native.ptr(ws), native.ptr(sd), Ns, T, Ns, Ks, code, limit,
                                       native.ptr(weigh_in), st), "experts_skinny")
        return parts
    tm = lib.hds_experts_gemm_tile(n, out_w, E) if fast else 64
    max_tiles = n // tm + min(E, n) + 1
    buf = torch.empty(E + 1 + 2 * n + 2 * max_tiles + 1, dtype=torch.int32, device=dev)
    offs, row, token, tile_e, tile_m, n_tiles = buf.split([E + 1, n, n, max_tiles, max_tiles, 1])
    row_weight = torch.empty(n, dtype=torch.float32, device=dev) if shape.weigh_input else None
    native.check(
        lib.hds_expert_sort(expert.data_ptr(), n, k, E, offs.data_ptr(), row.data_ptr(), token.data_ptr(),
                            native.ptr(weigh_in), native.ptr(row_weight), tm,
                            tile_e.data_ptr(), tile_m.data_ptr(), n_tiles.data_ptr(), max_tiles, st), "expert_sort")
    parts.row = row
    parts.y = torch.empty(n, out_w, dtype=x.dtype, device=dev)
    plan = (offs.data_ptr(), tile_e.data_ptr(), tile_m.data_ptr(), n_tiles.data_ptr(), max_tiles)
    if fast:
        h = torch.empty(n, inter, dtype=x.dtype, device=dev)
        native.check(
            lib.hds_experts_gemm(x.data_ptr(), x.stride(0), token.data_ptr(), T, w13.data_ptr(), h.data_ptr(), inter,
                                 *plan, tm, n, inter, K, E, 1, code, limit, native.ptr(row_weight), st), "experts_gemm")
        native.check(
            lib.hds_experts_gemm(h.data_ptr(), inter, None, 0, w2.data_ptr(), parts.y.data_ptr(), out_w, *plan, tm, n,
                                 out_w, inter, E, 0, 0, 0.0, None, st), "experts_gemm")
    else:
        gu = torch.empty(n, 2 * inter, dtype=x.dtype, device=dev)
        h = torch.empty(n, inter, dtype=x.dtype, device=dev)
        native.check(
            lib.hds_experts_gemm_f32(x.data_ptr(), x.stride(0), w13.data_ptr(), gu.data_ptr(), 2 * inter,
                                     token.data_ptr(), *plan, native.ptr(row_weight), n, 2 * inter, K, st),
            "experts_gemm_f32")
        glu_rows(gu, act, h, limit)
        native.check(
            lib.hds_experts_gemm_f32(h.data_ptr(), inter, w2.data_ptr(), parts.y.data_ptr(), out_w, None, *plan,
                                     None, n, out_w, inter, st), "experts_gemm_f32")
    if has_shared:
        parts.shared = _shared_product(x, w)
    return parts


def _routed_experts_cpu(x, w, shape, identity, act, limit):
    z = F.linear(x.float(), w["router.w"].float())
    expert, weight = route(z, w["router.c"], shape)
    y = torch.zeros(expert.numel(), w["w2"].shape[1], dtype=x.dtype)
    flat = expert.reshape(-1)
    for e in torch.unique(flat[flat < shape.experts]).tolist():
        a = (flat == e).nonzero()[:, 0]
        gu = F.linear(x[a // shape.top].float(), w["w13"][e].float())
        if shape.weigh_input:
            gu = gu * weight.reshape(-1, 1)[a]
        h = glu_rows(gu, act, torch.empty(gu.shape[0], gu.shape[1] // 2), limit)
        y[a] = F.linear(h.to(x.dtype).float(), w["w2"][e].float()).to(x.dtype)
    parts = ExpertSum(y, expert, None if shape.weigh_input else weight, None, shape.experts, identity=identity)
    if w["ws13"] is not None:
        parts.gate = z[:, shape.outputs]
        parts.shared = _shared_product(x, w)
    return parts
