"""Registered inference-v2 module implementations on the MI355X kernels
(reference inference/v2/modules/implementations/*: dense_blocked_attention, blas_fp_linear, quantized_linear
(wf6af16), cutlass_multi_gemm_moe, cuda_pre_rms / cuda_pre_ln / cuda_post_ln, ragged_embedding, ragged_unembed).

* attention: fused RoPE + paged-KV scatter and paged FlashAttention (csrc/kernels/paged_attn.hip, MFMA);
* linear: bf16 GEMM on hipBLASLt with the bias/activation epilogue in the HIP activation kernels; FP6 (e3m2) and
  INT8/INT4 weight-only variants read the packed weight straight from HBM at decode sizes (HIP GEMVs) and
  dequantize once per call for prefill-sized batches;
* MoE: sync-free top-k assignment + dropless grouped GEMM (csrc/kernels/grouped_gemm.hip);
* norms: the fused residual-add + RMSNorm / LayerNorm kernels (csrc/kernels/norm.hip).
"""
import torch
import torch.nn.functional as F

from .... import comm as dist
from ....ops.activations import bias_act, glu, glu_rows
from ....ops.delta_rule import DeltaShape, delta_rule, make_delta_plan, step_ok
from ....ops.experts import PAD, routed_experts
from ....ops.gated_scan import gated_scan, recur_step, recur_step_ok
from ....ops.gemv import glu_gemv
from ....ops.grouped_gemm import moe_ffn_dropless
from ....ops.head_prep import HeadPrep
from ....ops.input_norm import input_norm
from ....ops.latent_attention import LatentShape, can_expand, latent_attention, make_plan
from ....ops.matrix_memory import MemoryShape, make_memory_plan, matrix_memory
from ....ops.matrix_memory import step_ok as memory_step_ok
from ....ops.moe import moe_combine, moe_dispatch, topk_assign, topk_route
from ....ops.norm import layer_norm, rms_norm
from ....ops.output_norm import (PairSum, embed_rows, padded, residual_norm, rms_rows, sandwich_norm, softcap_,
                                 stream_norm, sum_experts)
from ....ops.paged import (HeadShape, head_attention, head_blocks_ok, kv_rope_scatter, make_head_plan,
                           paged_attention)
from ....ops.quantizer import fp6_linear, int_linear, quantize, quantize_minifloat
from ....ops.rope import rope_tables
from .interfaces import (DSEmbeddingBase, DSEmbeddingRegistry, DSExpertLayerBase, DSExpertLayerRegistry, DSGatedMLPBase,
                         DSGatedMLPRegistry, DSInputNormBase, DSInputNormRegistry, DSLinearBase, DSLinearRegistry,
                         DSMixerBase, DSMixerRegistry, DSMoEBase, DSMoERegistry, DSOutputNormBase, DSOutputNormRegistry,
                         DSPostNormBase, DSPostNormRegistry, DSPreNormBase, DSPreNormRegistry, DSSandwichNormBase,
                         DSSandwichNormRegistry, DSSelfAttentionBase, DSSelfAttentionRegistry, DSUnembedBase,
                         DSUnembedRegistry)

_PLAIN_ACTS = ("gelu", "gelu_tanh", "relu", "silu")


def _act_tail(y, bias, activation):
    """bias + activation epilogue shared by every linear implementation."""
    if activation == "identity":
        return y if bias is None else y + bias
    if activation.endswith("_glu"):
        return glu(y if bias is None else y + bias, activation[:-4])
    return bias_act(y, bias, activation)


def _supports_act(a):
    return a == "identity" or a in _PLAIN_ACTS or (a.endswith("_glu") and a[:-4] in _PLAIN_ACTS)


# ---------------------------------------------------------------------------------------------------------------
@DSSelfAttentionRegistry.register_module
class DSDenseBlockedAttention(DSSelfAttentionBase):

    @staticmethod
    def name():
        return "dense_blocked_attention"

    @staticmethod
    def supports_config(c):
        return c.n_heads_q % c.n_heads_kv == 0 and c.head_size % 16 == 0 and c.head_size <= 256

    def forward(self, qkv, cache, batch, cos, sin):
        c = self._config
        T = qkv.shape[0]
        nq, nkv, D = c.n_heads_q, c.n_heads_kv, c.head_size
        kv_rope_scatter(qkv, cache, batch.tok_seq, batch.tok_pos, batch.block_tables, cos, sin, nq, nkv,
                        do_rope=c.positional_embedding_type != "none" and cos is not None, rotary_dim=c.rotary_dim)
        o = paged_attention(qkv[:, :nq], cache, batch.atoms, batch.n_atoms, batch.seq_meta, batch.block_tables, nq,
                            nkv, c.scale_factor, c.sliding_window, batch.seq_meta_host, batch.tables_host,
                            decode=T == batch.current_sequences)
        return o.reshape(T, nq * D)


# ---------------------------------------------------------------------------------------------------------------
@DSLinearRegistry.register_module
class BlasFPLinear(DSLinearBase):

    @staticmethod
    def name():
        return "blas_fp_linear"

    @staticmethod
    def supports_config(c):
        return c.quantization_mode is None and _supports_act(c.activation)

    def forward(self, x, w, b=None):
        a = self._config.activation
        from ....ops.gemv import linear  # decode-sized ragged batches (<= 8 tokens) on the HIP GEMV
        if a == "identity" or a.endswith("_glu"):
            return _act_tail(linear(x, w, b), None, a)
        return bias_act(linear(x, w), b, a)


class _PackedWeight:
    """Weight-only quantized [out, in] matrix (groups along ``in``)."""

    def __init__(self, q, scales, out_features, in_features, group_size):
        self.q, self.scales = q, scales
        self.out_features, self.in_features, self.group_size = out_features, in_features, group_size
        self.shape = (out_features, in_features)

    def nbytes(self):
        return self.q.numel() * self.q.element_size() + self.scales.numel() * 4


def _group(c, in_features):
    g = c.group_size
    while in_features % g:
        g //= 2
    return g


@DSLinearRegistry.register_module
class QuantizedWf6Af16Linear(DSLinearBase):
    """FP6 (e3m2) weights, bf16 activations: the reference's ``quantized_wf6af16_linear``."""

    @staticmethod
    def name():
        return "quantized_wf6af16_linear"

    @staticmethod
    def supports_config(c):
        return c.quantization_mode == "wf6af16" and _supports_act(c.activation) and c.in_channels % 16 == 0

    def transform_param(self, w):
        if isinstance(w, _PackedWeight) or w is None:
            return w
        out_f, in_f = w.shape
        g = _group(self._config, in_f)
        q, s = quantize_minifloat(w.contiguous(), g, 6, 2)
        return _PackedWeight(q, s, out_f, in_f, g)

    def forward(self, x, w, b=None):
        y = fp6_linear(x, w.q, w.scales, w.out_features, w.in_features, w.group_size, 2)
        return _act_tail(y, b, self._config.activation)


@DSLinearRegistry.register_module
class QuantizedIntLinear(DSLinearBase):
    """Symmetric group-wise INT8 / INT4 weights, bf16 activations (inference v1's int8 weight path in v2)."""

    @staticmethod
    def name():
        return "quantized_int_linear"

    @staticmethod
    def supports_config(c):
        return c.quantization_mode in ("int8", "int4") and _supports_act(c.activation) and c.in_channels % 16 == 0

    def _bits(self):
        return 8 if self._config.quantization_mode == "int8" else 4

    def transform_param(self, w):
        if isinstance(w, _PackedWeight) or w is None:
            return w
        out_f, in_f = w.shape
        g = _group(self._config, in_f)
        q, s, _ = quantize(w.contiguous(), g, self._bits(), True)
        return _PackedWeight(q, s, out_f, in_f, g)

    def forward(self, x, w, b=None):
        y = int_linear(x, w.q, w.scales, w.out_features, w.in_features, w.group_size, self._bits())
        return _act_tail(y, b, self._config.activation)


# ---------------------------------------------------------------------------------------------------------------
@DSMoERegistry.register_module
class GroupedGemmMoE(DSMoEBase):
    """Top-k MoE without token dropping. GPU bf16: sync-free routing + two HIP grouped GEMMs over the
    expert-contiguous rows; elsewhere: capacity slots + batched expert GEMMs."""

    @staticmethod
    def name():
        return "grouped_gemm_moe"

    @staticmethod
    def supports_config(c):
        return c.activation.endswith("_glu") and 1 <= c.top_k <= c.n_experts

    def forward(self, x, router_w, w13, w2):
        c = self._config
        act = c.activation[:-4]
        T, H = x.shape
        logits = F.linear(x.float(), router_w.float())
        if x.is_cuda and x.dtype == torch.bfloat16 and H % 128 == 0 and w2.shape[2] % 128 == 0:
            expert, pos, w, counts = topk_assign(logits, c.top_k, normalize=c.normalize_scores)
            return moe_ffn_dropless(x, expert, pos, w, counts, w13, w2, lambda h: glu(h, act))
        E = logits.shape[-1]
        expert, pos, w, C, _, _ = topk_route(logits, c.top_k, 1.0, 1, drop_tokens=False, use_rts=False,
                                             normalize=c.normalize_scores, training=False)
        disp = moe_dispatch(x, expert, pos, E, C).view(E, C, H)
        from ....parallel.moe import expert_linear  # per-expert 2-D GEMMs on the GPU (see its docstring)
        with torch.no_grad():
            h = expert_linear(disp, w13)
            y = expert_linear(glu(h.reshape(E * C, -1), act).view(E, C, -1), w2)
        return moe_combine(y.reshape(E * C, H), expert, pos, w, C)


# ---------------------------------------------------------------------------------------------------------------
@DSPreNormRegistry.register_module
class DSPreRMSNorm(DSPreNormBase):

    @staticmethod
    def name():
        return "ds_pre_rms"

    @staticmethod
    def supports_config(c):
        return c.type == "rms"

    def forward(self, residual, hidden_in, gamma, beta=None):
        if hidden_in is None:
            return residual, rms_norm(residual, gamma, self._config.eps)
        y, r = rms_norm(hidden_in, gamma, self._config.eps, residual)
        return r, y


@DSPreNormRegistry.register_module
class DSPreLayerNorm(DSPreNormBase):

    @staticmethod
    def name():
        return "ds_pre_ln"

    @staticmethod
    def supports_config(c):
        return c.type == "layer"

    def forward(self, residual, hidden_in, gamma, beta=None):
        if hidden_in is None:
            return residual, layer_norm(residual, gamma, beta, self._config.eps)
        y, r = layer_norm(hidden_in, gamma, beta, self._config.eps, residual)
        return r, y


@DSPostNormRegistry.register_module
class DSPostLayerNorm(DSPostNormBase):

    @staticmethod
    def name():
        return "ds_post_ln"

    @staticmethod
    def supports_config(c):
        return c.type in ("layer", "rms")

    def forward(self, residual, hidden_in, gamma, beta=None):
        if self._config.type == "rms":
            y, _ = rms_norm(hidden_in, gamma, self._config.eps, residual)
        else:
            y, _ = layer_norm(hidden_in, gamma, beta, self._config.eps, residual)
        return y


# ---------------------------------------------------------------------------------------------------------------
@DSEmbeddingRegistry.register_module
class RaggedEmbedding(DSEmbeddingBase):

    @staticmethod
    def name():
        return "ragged_embedding"

    def forward(self, batch, word_embeddings, position_embeddings=None):
        h = F.embedding(batch.input_ids, word_embeddings)
        if position_embeddings is not None:
            h = h + F.embedding(batch.tok_pos.long() + self._config.positional_offset, position_embeddings)
        return h


@DSUnembedRegistry.register_module
class RaggedUnembed(DSUnembedBase):
    """Gathers each sequence's last token, applies the final norm (fused residual add) and the vocab GEMM; under
    TP the vocab is sharded by rows and the shards are all-gathered."""

    @staticmethod
    def name():
        return "ragged_unembed"

    def forward(self, hidden, residual, batch, lm_head, lm_head_b, final_w, final_b, norm_eps=1e-5, tp_group=None,
                vocab=None):
        idx = batch.last_token_idx
        if final_w is not None:
            if self._config.norm_type == "rms":
                hl, _ = rms_norm(hidden[idx], final_w, norm_eps, residual[idx])
            else:
                hl, _ = layer_norm(hidden[idx], final_w, final_b, norm_eps, residual[idx])
        else:
            hl = hidden[idx] + residual[idx]
        return self.project(hl, lm_head, lm_head_b, tp_group, vocab)

    def project(self, hl, lm_head, lm_head_b=None, tp_group=None, vocab=None):
        """Logits of already normed rows."""
        logits = F.linear(hl, lm_head, lm_head_b)
        tp = dist.get_world_size(tp_group) if tp_group is not None else 1
        if tp > 1:
            parts = [torch.empty_like(logits) for _ in range(tp)]
            dist.all_gather(parts, logits, group=tp_group)
            logits = torch.cat(parts, -1)[:, :vocab].contiguous()
        return softcap_(logits, self._config.softcap) if self._config.softcap else logits


# ---------------------------------------------------------------------------------------------------------------
# layers with a 32-bit residual stream and mixers of several kinds
# ---------------------------------------------------------------------------------------------------------------
@DSInputNormRegistry.register_module
class RmsInputConv(DSInputNormBase):
    """Residual add, RMS norm with scalar or vector gains and a causal input convolution per sublayer, one kernel."""

    @staticmethod
    def name():
        return "rms_input_conv"

    @staticmethod
    def supports_config(c):
        return c.type == "rms" and 1 <= c.conv_taps <= 16

    def state_floats(self):
        n = (self._config.conv_taps - 1) * self._config.channels
        return -(-n // 4) * 4

    def forward(self, x, delta, gains, convs, batch, state, offset, embed=None):
        c = self._config
        return input_norm(x, delta, gains, convs, c.eps, c.conv_taps, batch, state, offset, c.input_dtype, embed)


def _is_plain(lin):
    return isinstance(lin, BlasFPLinear)


SPLIT_ROWS = 1024  # tokens from which on a projection may run as several products


def _tile_rounds(rows, cols):
    """How often the library's 256 x 256 tiles of a product go round the 256 CUs."""
    return -(-(-(-rows // 256) * -(-cols // 256)) // 256)


@DSMixerRegistry.register_module
class MinGRUMixer(DSMixerBase):
    """Gated linear recurrence whose gates read the current token only (ops/gated_scan.py)."""

    FUSED_ROWS = 4  # decode batches of at most this many sequences run projection and recurrence in one kernel

    @staticmethod
    def name():
        return "mingru"

    def __init__(self, config, implementation_config=None):
        super().__init__(config, implementation_config)
        assert config.params["width"] % config.tp == 0, "the recurrence's width must divide the tensor-parallel size"
        self.width = self.out_width = config.params["width"] // config.tp
        self.in_width = 3 * self.width

    def state_floats(self):
        return -(-self.width // 4) * 4

    def shard(self, w, rows, cols):
        return {"in.w": torch.cat([rows(w["z"]), rows(w["x"]), rows(w["g"])]), "o.w": cols(w["o"]),
                "z.b": rows(w["z.b"]).float(), "x.b": rows(w["x.b"]).float()}

    def forward(self, x, w, lins, out, batch, cache, state, offset):
        lin = lins["in.w"]
        if batch.max_new == 1 and _is_plain(lin) and recur_step_ok(x, w["in.w"], self.FUSED_ROWS) and \
                x.shape[0] == batch.current_sequences:
            return recur_step(x, w["in.w"], w["z.b"], w["x.b"], out, batch, state, offset)
        return gated_scan(lin(x, w["in.w"]), w["z.b"], w["x.b"], out, batch, state, offset)


def _pair_order(rot_dims, dim):
    """Dimensions of a head whose halves i and i + rot_dims / 2 turn together, in the order the kernels turn them in."""
    return [i for j in range(rot_dims // 2) for i in (j, j + rot_dims // 2)] + list(range(rot_dims, dim))


def _lone_plan(kind, batch, single, make):
    """The batch's plan of lone tokens and portions for a kind of recurrence (shared by layers of the same answer)."""
    key = (kind, single)
    plan = batch.plans.get(key)
    if plan is None:
        plan = batch.plans[key] = make(batch.seq_meta_host, batch.current_sequences, batch.max_new, single,
                                       batch.tok_pos.device)
    return plan


@DSMixerRegistry.register_module
class LatentAttentionMixer(DSMixerBase):
    """Attention over compressed K/V rows, sliding window, rotation of a shared key part, optionally queries through a
    latent of their own and a gate per head (ops/latent_attention.py). Heads are sharded over the tensor-parallel group,
    the latents are computed on every rank. The kernels turn neighbouring dimensions; the "half" rotation, which pairs i
    with i + rot_dims / 2, becomes that by reordering the rotated rows of the query and key weights."""

    @staticmethod
    def name():
        return "latent_attention"

    def __init__(self, config, implementation_config=None):
        super().__init__(config, implementation_config)
        p = config.params
        assert p["heads"] % config.tp == 0, "attention heads must divide the tensor-parallel size"
        self.shape = LatentShape(heads=p["heads"] // config.tp, dim=p["dim"], rot=p["rot_dim"], rot_dims=p["rot_dims"],
                                 rank=p["kv_rank"], vdim=p["vdim"], window=p["window"], scale=p["scale"],
                                 eps=config.eps, gated=p.get("gated", False))
        self.rope_base, self.rope_scaling = p["rope_base"], p.get("rope_scaling")
        self.half = p.get("rot_layout", "interleaved") == "half"
        self.q_rank = p.get("q_rank", 0)  # 0: queries straight from the input
        self.out_width = self.shape.heads * self.shape.vdim
        self.width = (self.q_rank or self.shape.q_width) + self.shape.row + (self.shape.heads if self.shape.gated else 0)
        self.in_width = padded(self.width, 8) if self.q_rank or self.shape.gated else self.width
        self.cache_row = self.shape.row
        self.cos = self.sin = None

    def extra_linears(self):
        return {"uq.w": (self.q_rank, self.shape.q_width)} if self.q_rank else {}

    def _turned(self, w):
        """w [..., rot, in]: the rotated rows in the kernels' order."""
        return w[..., _pair_order(self.shape.rot_dims, self.shape.rot), :] if self.half else w

    def bind_tables(self, cos, sin):
        self.cos, self.sin = cos, sin

    def bind_positions(self, positions, device):
        self.bind_tables(*rope_tables(positions, self.shape.rot_dims, self.rope_base, self.rope_scaling, device=device))

    def shard(self, w, rows, cols):
        # q, uk, uv and the gate are laid out head by head: equal row slices are whole heads
        sh = self.shape
        q = rows(w["uq"] if self.q_rank else w["q"])
        q = q.reshape(sh.heads, sh.dim + sh.rot, -1)
        q = torch.cat([q[:, :sh.dim], self._turned(q[:, sh.dim:])], 1).reshape(sh.q_width, -1)
        parts = [w["dq"] if self.q_rank else q, w["dkv"][:sh.rank], self._turned(w["dkv"][sh.rank:])]
        if sh.gated:
            parts.append(rows(w["g"]))
        out = {"o.w": cols(w["o"]), "ukv.w": torch.cat([rows(w["uk"]), rows(w["uv"])]),
               "dkv.norm": w["dkv.norm"].float()}
        if self.q_rank:
            out["uq.w"], out["dq.norm"] = q, w["dq.norm"].float()
        if self.in_width > self.width:
            parts.append(q.new_zeros(self.in_width - self.width, parts[0].shape[1]))
        out["in.w"] = torch.cat(parts)
        return out

    def _plan(self, batch):
        sh = self.shape
        if batch.max_new == 1:
            expand = False
        else:
            expand = can_expand(sh, self._config.input_dtype) if batch.tok_pos.is_cuda else False
        key = (sh.window, expand)
        plan = batch.plans.get(key)
        if plan is None:
            plan = batch.plans[key] = make_plan(batch.seq_meta_host if expand else [], batch.current_tokens, sh.window,
                                                expand, batch.tok_pos.device)
        return plan

    def forward(self, x, w, lins, out, batch, cache, state, offset):
        sh = self.shape
        ukv = w["ukv.w"]
        uk = ukv[:sh.heads * sh.dim].view(sh.heads, sh.dim, sh.rank)
        uv = ukv[sh.heads * sh.dim:].view(sh.heads, sh.vdim, sh.rank)
        y = lins["in.w"](x, w["in.w"])
        n = self.q_rank or sh.q_width
        q, ckr = y[:, :n], y[:, n:n + sh.row]
        gate = y[:, n + sh.row:self.width] if sh.gated else None
        if self.q_rank:
            q = lins["uq.w"](rms_rows(q, w["dq.norm"], sh.eps), w["uq.w"])
        return latent_attention(q, ckr, sh, w["dkv.norm"], uk, uv, ukv, self.cos, self.sin, cache, batch,
                                self._plan(batch), out, gate)


@DSMixerRegistry.register_module
class HeadAttentionMixer(DSMixerBase):
    """Grouped-query attention: sliding window (the sequence's first ``keep`` tokens stay visible) or chunks, soft cap, sink
    (learned or of score zero), output gate per head or element, and values mixed with those of an earlier layer
    (``value_mix``: "source" leaves its values for the later ones of the step, "mix" takes them). Queries and keys are normed
    head by head, if at all; or, with ``conv`` in the parameters, convolved over a few tokens, normed across all heads
    (``norm_all``) and rotated (``rot_dims``, neighbouring pairs), and the keys as convolved may be the values
    (``shared_values``). ops/paged.py ``head_attention``. Heads are sharded over the tensor-parallel group."""

    @staticmethod
    def name():
        return "attention"

    def __init__(self, config, implementation_config=None):
        super().__init__(config, implementation_config)
        p, tp = config.params, config.tp
        if p["heads"] % tp or p["kv_heads"] % tp or p["heads"] % p["kv_heads"]:
            raise ValueError(f"{p['heads']} / {p['kv_heads']} heads: not groups of equal size on {tp} ranks")
        self.shape = HeadShape(heads=p["heads"] // tp, kv_heads=p["kv_heads"] // tp, dim=p["dim"], vdim=p["vdim"],
                               window=p["window"], scale=p["scale"], eps=config.eps, gated=p["gated"],
                               gate_width=p["vdim"] if p.get("gate_elements") else 1, chunk=p.get("chunk", 0),
                               softcap=p.get("softcap", 0.0), keep=p.get("keep", 0), prep="conv" in p,
                               taps=p.get("conv", 1), rot=p.get("rot_dims", 0), shared=p.get("shared_values", False))
        self.norm_all = p.get("norm_all", False)
        self.rope_base, self.rope_scaling = p.get("rope_base"), p.get("rope_scaling")
        self.tables = self.reduce = None
        self.value_mix = p.get("value_mix")
        self.zero_sink = p.get("zero_sink", False)
        self.out_width = self.shape.heads * p["vdim"]
        self.in_width = padded(self.shape.width, 8)  # 16-byte rows
        self.cache_row = self.shape.row

    def state_floats(self):
        return padded(self.shape.state_floats, 4)

    def bind_positions(self, positions, device):
        if self.shape.rot:
            self.tables = rope_tables(positions, self.shape.rot, self.rope_base, self.rope_scaling, device=device)

    def bind_group(self, reduce):
        self.reduce = reduce

    def shard(self, w, rows, cols):
        # q, k, v, g, convolutions, norms across heads and the sink are laid out head by head: equal slices are whole heads
        names = ["q", "k"] + (["v"] if not self.shape.shared else []) + (["g"] if self.shape.gated else [])
        parts = [rows(w[k]) for k in names]
        fill = self.in_width - self.shape.width
        if fill:
            parts.append(parts[0].new_zeros(fill, parts[0].shape[1]))
        out = {"in.w": torch.cat(parts), "o.w": cols(w["o"])}
        for k in ("q.norm", "k.norm"):
            out[k] = (rows(w[k]) if self.norm_all else w[k]).float() if k in w else None
        if self.shape.prep:
            conv = [w.get("q.conv"), w.get("k.conv")]
            out["conv.w"] = None if conv[0] is None else torch.cat([rows(c) for c in conv]).float().t().contiguous()
        out["sink"] = rows(w["sink"]).float() if "sink" in w else None
        if self.zero_sink:
            out["sink"] = torch.zeros(self.shape.heads)
        if self.value_mix == "mix":
            out["vmix"] = w["vmix"].reshape(1).float()
        return out

    def _plan(self, batch):
        sh = self.shape
        blocks = batch.max_new > 1 and batch.tok_pos.is_cuda and head_blocks_ok(sh, self._config.input_dtype)
        key = ("heads", sh.heads, sh.kv_heads, blocks)
        plan = batch.plans.get(key)
        if plan is None:
            plan = batch.plans[key] = make_head_plan(batch.seq_meta_host if blocks else [], batch.current_tokens,
                                                     sh.heads, sh.kv_heads, blocks, batch.tok_pos.device)
        return plan

    def forward(self, x, w, lins, out, batch, cache, state, offset):
        sh = self.shape
        lin, in_w, n = lins["in.w"], w["in.w"], sh.qkv_width
        gate = None
        if sh.gate_width > 1 and x.shape[0] >= SPLIT_ROWS and _is_plain(lin) and n % 8 == 0:
            # gates as wide as the heads: of two narrower products both are closer to the library's best
            qkv, gate = lin(x, in_w[:n]), lin(x, in_w[n:sh.width])
        else:
            qkv = lin(x, in_w)
        return self.mix(qkv, w, out, batch, cache, state, offset, gate)

    def mix(self, qkv, w, out, batch, cache, state, offset, gate=None):
        """The projected rows (``gate``: without the gates) -> the heads' outputs."""
        sh = self.shape
        if sh.prep:
            prep = HeadPrep(w["conv.w"], w["q.norm"], w["k.norm"], self.tables, state, offset, self._config.tp, self.reduce)
            return head_attention(qkv, sh, None, None, w["sink"], cache, batch, self._plan(batch), out, gate=gate, prep=prep)
        own = qkv[:, sh.qkv_width - sh.kv_heads * sh.vdim:sh.qkv_width]
        if self.value_mix == "source":
            batch.carry["values"] = own
        first = batch.carry["values"] if self.value_mix == "mix" else None
        return head_attention(qkv, sh, w["q.norm"], w["k.norm"], w["sink"], cache, batch, self._plan(batch), out, first,
                              w["vmix"], gate)


@DSMixerRegistry.register_module
class DeltaMixer(DSMixerBase):
    """Gated delta rule with short convolutions (ops/delta_rule.py). Heads are sharded over the tensor-parallel group."""

    @staticmethod
    def name():
        return "delta"

    def __init__(self, config, implementation_config=None):
        super().__init__(config, implementation_config)
        p, tp = config.params, config.tp
        if p["heads"] % tp or p["kv_heads"] % tp or p["heads"] % p["kv_heads"]:
            raise ValueError(f"{p['heads']} / {p['kv_heads']} heads: not groups of equal size on {tp} ranks")
        self.shape = DeltaShape(heads=p["heads"] // tp, kv_heads=p["kv_heads"] // tp, dim=p["dim"], vdim=p["vdim"],
                                taps=p["conv"], eps=config.eps)
        self.out_width = self.shape.heads * self.shape.vdim
        self.in_width = padded(self.shape.width, 8)

    def state_floats(self):
        return padded(self.shape.state_floats, 4)

    def shard(self, w, rows, cols):
        # everything is laid out head by head: equal slices are whole heads
        parts = [rows(w[k]) for k in ("q", "k", "v", "g", "b", "a")]
        fill = self.in_width - self.shape.width
        if fill:
            parts.append(parts[0].new_zeros(fill, parts[0].shape[1]))
        conv = torch.cat([rows(w[k + ".conv"]) for k in ("q", "k", "v")])
        return {"in.w": torch.cat(parts), "o.w": cols(w["o"]), "conv.w": conv.float().t().contiguous(),
                "A_log": rows(w["A_log"]).float(), "dt_bias": rows(w["dt_bias"]).float(), "norm": w["norm"].float()}

    def _plan(self, batch):
        return _lone_plan("delta", batch, batch.tok_pos.is_cuda and step_ok(self.shape), make_delta_plan)

    def forward(self, x, w, lins, out, batch, cache, state, offset):
        sh, lin, in_w, T = self.shape, lins["in.w"], w["in.w"], x.shape[0]
        n, ba = sh.main_width, None
        if T >= SPLIT_ROWS and _is_plain(lin) and n % 8 == 0 and _tile_rounds(T, n) < _tile_rounds(T, self.in_width):
            # the few columns of b and a would cost another round of tiles
            proj, ba = lin(x, in_w[:n]), lin(x, in_w[n:])
        else:
            proj = lin(x, in_w)
        return delta_rule(proj, sh, w["conv.w"], w["A_log"], w["dt_bias"], w["norm"], state, offset, batch,
                          self._plan(batch), out, ba)


class _MatrixMemoryMixer(DSMixerBase):
    """Linear attention with a decaying matrix state per head (ops/matrix_memory.py). Heads are sharded over the
    tensor-parallel group. The kernels turn neighbouring dimensions; the "half" rotation becomes that by reordering the
    rotated rows of the query and key weights."""

    def _init(self, **kind):
        p, c = self._config.params, self._config
        if p["heads"] % c.tp:
            raise ValueError(f"{p['heads']} heads: not groups of equal size on {c.tp} ranks")
        self.shape = MemoryShape(heads=p["heads"] // c.tp, dim=p["dim"], vdim=p["vdim"], eps=c.eps,
                                 rot=p.get("rot_dims", 0), **kind)
        self.half = p.get("rot_layout", "interleaved") == "half"
        self.rope_base, self.rope_scaling = p.get("rope_base"), p.get("rope_scaling")
        self.out_width = self.shape.heads * self.shape.vdim
        self.in_width = padded(self.shape.width, 8)
        self.tables = None

    def state_floats(self):
        return padded(self.shape.state_floats, 4)

    def bind_positions(self, positions, device):
        if self.shape.rot:
            self.tables = rope_tables(positions, self.shape.rot, self.rope_base, self.rope_scaling, device=device)

    def _turned(self, w):
        """w [heads * dim, in]: the rotated rows of every head in the kernels' order."""
        sh = self.shape
        if not (sh.rot and self.half):
            return w
        return w.reshape(sh.heads, sh.dim, -1)[:, _pair_order(sh.rot, sh.dim)].reshape(sh.heads * sh.dim, -1)

    def _extra(self, w, rows):
        """Further weights, and the rows of the input projection behind the output gate."""
        raise NotImplementedError

    def shard(self, w, rows, cols):
        # everything is laid out head by head: equal slices are whole heads
        extra, gates = self._extra(w, rows)
        parts = [self._turned(rows(w["q"])), self._turned(rows(w["k"])), rows(w["v"]), rows(w["g"])] + gates
        fill = self.in_width - self.shape.width
        if fill:
            parts.append(parts[0].new_zeros(fill, parts[0].shape[1]))
        return {"in.w": torch.cat(parts), "o.w": cols(w["o"]), **extra}

    def forward(self, x, w, lins, out, batch, cache, state, offset):
        return self.mix(lins["in.w"](x, w["in.w"]), w, out, batch, cache, state, offset)

    def mix(self, proj, w, out, batch, cache, state, offset):
        """The projected rows -> the heads' outputs."""
        plan = _lone_plan("memory", batch, batch.tok_pos.is_cuda and memory_step_ok(self.shape), make_memory_plan)
        return matrix_memory(proj, self.shape, w, self.tables, state, offset, batch, plan, out)


@DSMixerRegistry.register_module
class MLSTMMixer(_MatrixMemoryMixer):
    """Exponential input and forget gates with soft caps, a normalizer, a norm weight across all heads, a sigmoid gate."""

    @staticmethod
    def name():
        return "mlstm"

    def __init__(self, config, implementation_config=None):
        super().__init__(config, implementation_config)
        self._init(gate="sigmoid", gated=True, cap=config.params["cap"])

    def _extra(self, w, rows):
        extra = {"norm": rows(w["norm"]).float(), "i.b": rows(w["i.b"]).float(), "f.b": rows(w["f.b"]).float()}
        return extra, [rows(w["i"]), rows(w["f"])]


@DSMixerRegistry.register_module
class RetentionMixer(_MatrixMemoryMixer):
    """A fixed decay per head, rotated queries and keys, a norm without weights, a SiLU gate."""

    @staticmethod
    def name():
        return "retention"

    def __init__(self, config, implementation_config=None):
        super().__init__(config, implementation_config)
        self._init(gate="silu", gated=False)

    def _extra(self, w, rows):
        decay = torch.tensor(self._config.params["decay"], dtype=torch.float64).clamp(min=1e-38)
        return {"log_decay": rows(decay.log().float()), "norm": None}, []


class _Part:
    """The entries of a layer's weights that share a prefix."""

    def __init__(self, w, prefix):
        self.w, self.prefix = w, prefix

    def __getitem__(self, k):
        return self.w[self.prefix + k]


@DSMixerRegistry.register_module
class ParallelMixer(DSMixerBase):
    """Two mixers that read the same rows: one input projection, an output projection each, and the mean of both outputs,
    each RMS-normed over the model width."""
    own_output = True
    SIDES = ("left", "right")

    @staticmethod
    def name():
        return "parallel"

    def __init__(self, config, implementation_config=None):
        super().__init__(config, implementation_config)
        c = config
        self.parts = []
        for side in self.SIDES:
            p = c.params[side]
            cls = DSMixerRegistry.registry[p["type"]]
            self.parts.append(cls(type(c)(p["type"], c.model_dim, p, c.eps, c.tp, c.input_dtype), implementation_config))
        self.in_width = sum(m.in_width for m in self.parts)
        self.out_width = sum(m.out_width for m in self.parts)
        if sum(m.cache_row > 0 for m in self.parts) > 1:
            raise NotImplementedError("two cached mixers side by side")
        self.cache_row = sum(m.cache_row for m in self.parts)

    def state_floats(self):
        return sum(m.state_floats() for m in self.parts)

    def bind_positions(self, positions, device):
        for m in self.parts:
            m.bind_positions(positions, device)

    def bind_group(self, reduce):
        for m in self.parts:
            m.bind_group(reduce)

    def extra_linears(self):
        return {f"{s}.o.w": (m.out_width, self._config.model_dim) for s, m in zip(self.SIDES, self.parts)}

    def shard(self, w, rows, cols):
        out, ins = {}, []
        for side, m in zip(self.SIDES, self.parts):
            own = m.shard({k[len(side) + 1:]: v for k, v in w.items() if k.startswith(side + ".")}, rows, cols)
            ins.append(own.pop("in.w"))
            out.update({f"{side}.{k}": v for k, v in own.items()})
            out[f"{side}.out"] = w[side + ".out"].float()
        return {"in.w": torch.cat(ins), **out}

    def forward(self, x, w, lins, out, batch, cache, state, offset):
        y = lins["in.w"](x, w["in.w"])
        i = o = 0
        for side, m in zip(self.SIDES, self.parts):
            m.mix(y[:, i:i + m.in_width], _Part(w, side + "."), out[:, o:o + m.out_width], batch,
                  cache if m.cache_row else None, state, offset)
            i, o, offset = i + m.in_width, o + m.out_width, offset + m.state_floats()

    def output(self, mid, w, lins, reduce):
        y, o = [], 0
        for side, m in zip(self.SIDES, self.parts):
            y.append(reduce(lins[f"{side}.o.w"](mid[:, o:o + m.out_width], w[f"{side}.o.w"])))
            o += m.out_width
        return PairSum(*y, w["left.out"], w["right.out"])


@DSOutputNormRegistry.register_module
class RmsResidual(DSOutputNormBase):
    """32-bit residual, RMS norm of what is added to it; bf16 rows come zero-padded to the expert products' tile."""

    @staticmethod
    def name():
        return "rms_residual"

    @staticmethod
    def supports_config(c):
        return c.type == "rms"

    def _pad(self):
        return PAD if self._config.input_dtype == torch.bfloat16 else 1

    def start(self, embed, ids, scale):
        return embed_rows(embed, ids, scale, self._config.input_dtype, self._pad())

    def forward(self, x, delta, gain):
        return residual_norm(x, delta, gain, self._config.eps, self._config.input_dtype, self._pad())


@DSSandwichNormRegistry.register_module
class RmsSandwich(DSSandwichNormBase):
    """32-bit residual, RMS norms on both sides of every sublayer; the step between two sublayers is one kernel."""

    @staticmethod
    def name():
        return "rms_sandwich"

    @staticmethod
    def supports_config(c):
        return c.type == "rms"

    def forward(self, x, delta, norm, next_norm, embed=None, idx=None, pad=1):
        assert pad == 1
        return sandwich_norm(x, delta, norm, next_norm, self._config.eps, self._config.input_dtype, embed, idx)


@DSSandwichNormRegistry.register_module
class LnSandwich(DSSandwichNormBase):
    """32-bit residual, layer norms on both sides of every sublayer (RMS norms where only a gain is given)."""

    @staticmethod
    def name():
        return "ln_sandwich"

    @staticmethod
    def supports_config(c):
        return c.type == "layer"

    def forward(self, x, delta, norm, next_norm, embed=None, idx=None, pad=1):
        dt = self._config.input_dtype
        if x is None:
            x = embed_rows(*embed, dt)[0]
        return stream_norm(x, delta, norm, next_norm, self._config.eps, dt, idx, pad)


@DSExpertLayerRegistry.register_module
class RoutedExperts(DSExpertLayerBase):
    """Top-k experts, optionally limited to groups, with identity experts and a gated shared expert (ops/experts.py). Every expert's
    feed-forward width is sharded over the tensor-parallel group; bf16 weights are zero-padded to the products' tile."""

    @staticmethod
    def name():
        return "routed_experts"

    def __init__(self, config, implementation_config=None):
        super().__init__(config, implementation_config)
        config.router.check()
        if config.intermediate_features % config.tp or config.shared_features % config.tp:
            raise ValueError("the experts' widths must divide the tensor-parallel size")

    def row_pad(self):
        """What the length of the rows it reads has to be a multiple of."""
        return PAD if self._config.input_dtype == torch.bfloat16 else 1

    def _fit(self, w):
        """w zero-padded at the end of its last two dimensions."""
        if self._config.input_dtype != torch.bfloat16:
            return w
        add = [padded(n, PAD) - n for n in w.shape[-2:]]
        return F.pad(w, (0, add[1], 0, add[0])) if any(add) else w

    def _gate_up(self, gate, up, rows):
        # ``rows`` slices the first dimension
        gate, up = (rows(t.transpose(0, -2)).transpose(0, -2) for t in (gate, up))
        return torch.cat([self._fit(gate), self._fit(up)], -2)

    def shard(self, w, rows, cols):
        fit, shared = self._fit, self._config.shared_features > 0
        router = torch.cat([w["router"], w["shared.sg"]]) if shared else w["router"]
        n = router.shape[0]
        correction = w["correction"].float() if "correction" in w else None
        return {"router.w": fit(router)[:n], "router.c": correction,
                "w13": self._gate_up(w["gate"], w["up"], rows), "w2": fit(cols(w["down"])),
                "ws13": self._gate_up(w["shared.gate"], w["shared.up"], rows) if shared else None,
                "ws2": fit(cols(w["shared.down"])) if shared else None}

    def forward(self, x, w, rank=0):
        c = self._config
        return routed_experts(x, w, c.router, identity=rank == 0, act=c.activation, limit=c.limit)

    def total(self, x32, parts):
        return sum_experts(x32, parts, self._config.input_dtype)


@DSGatedMLPRegistry.register_module
class GatedMLPRows(DSGatedMLPBase):
    """act(x gate^T) * (x up^T), or the clamped unit, into a column block: one GEMV for decode rows, else projection +
    activation kernel."""

    FUSED_ROWS = 1

    @staticmethod
    def name():
        return "gated_mlp_rows"

    @staticmethod
    def supports_config(c):
        return c.activation in _PLAIN_ACTS + ("clamped", )

    def forward(self, x, w, lin, out):
        act, limit = self._config.activation, self._config.limit
        if x.shape[0] <= self.FUSED_ROWS and _is_plain(lin) and glu_gemv(x, w, act, out, limit):
            return out
        return glu_rows(lin(x, w), act, out, limit)
