"""Decoders whose layers are listed one by one in :class:`arch.ArchSpec` ``layers``: mixers of several kinds, layers that
run more than once with the same weights (``loop`` / ``order``), a 32-bit residual stream. Served by the same engine,
paged cache, batch metadata and decode graphs as :class:`model.RaggedTransformer`. Three layer forms:

* :class:`HybridTransformer` (``norm_place`` "pre"): mixer and gated MLP read the same residual (parallel block, two
  norms), with a causal convolution in front of every sublayer. A layer is: input norm (residual add + norm +
  convolutions, one kernel), the mixer and the gated MLP into two column blocks of one matrix, and ONE output projection
  [W_o | W_down] of that matrix;
* :class:`PostNormTransformer` ("post"): mixer, then expert layer, each reading the residual itself; the norm is on their
  outputs. A layer is: mixer and its output projection, norm + residual add (one kernel), router and experts, and one
  kernel that sums the experts' outputs, norms the sum and adds it.
* :class:`SandwichTransformer` ("both"): mixer, then gated MLP or routed experts, each between a norm of its input and a norm
  of its output (RMS or layer norms). One kernel between two sublayers norms the first one's output, adds it to the residual
  and norms the sum for the next. Optionally a third sublayer without a norm of its input: the residual gates a row of the
  token's own, one per layer (``token_side``), and a second embedding row by the previous and this token (``pair_embed``).

Common to all:

* every layer *run* (a pass of a looped or shared layer counts) has its own paged cache rows and its own part of the sequence's
  state row (``ragged.SequenceStatePool``): convolution tails and recurrent states, float32;
* HCache latents are the attention runs' cached rows themselves, side by side ([1, tokens, sum of row widths]): they
  are already the compressed form. ``restore_kv`` scatters them back; the state row travels with ``evict``.
"""
import torch

from ...ops.activations import act_gather
from ...ops.experts import RouterShape
from ...ops.gemv import gather_gemv
from ...ops.output_norm import embed_pairs, norm_rows
from ...ops.paged import copy_rows
from .arch import run_order
from .model import RaggedTransformer, _Layer
from .modules import (DSExpertLayerConfig, DSGatedMLPConfig, DSInputNormConfig, DSLinearConfig, DSMixerConfig,
                      DSNormConfig, DSUnembedConfig, instantiate_expert_layer, instantiate_gated_mlp,
                      instantiate_input_norm, instantiate_linear, instantiate_mixer, instantiate_output_norm,
                      instantiate_sandwich_norm, instantiate_unembed)
from .modules.implementations import BlasFPLinear, _PackedWeight


class _Run:
    """One pass of one layer: where its cached rows and its states are."""
    __slots__ = ("layer", "cache", "tail", "state")

    def __init__(self, layer, cache, tail, state):
        self.layer, self.cache, self.tail, self.state = layer, cache, tail, state


# weights kept in the engine's dtype; every other float32 tensor stays float32
_MATRICES = ("in.w", "up.w", "out.w", "down.w", "uq.w", "ukv.w", "router.w", "w13", "w2", "ws13", "ws2", "left.o.w",
             "right.o.w", "side.gate.w", "side.proj.w")


class HybridTransformer(RaggedTransformer):
    # kernel sources this class runs on, for builds of just those (ops/build.py)
    KERNEL_SOURCES = ("act.hip", "gated_scan.hip", "gemv.hip", "input_norm.hip", "latent_attn.hip", "output_norm.hip",
                      "paged_rows.hip")

    def __init__(self, spec, weights, device, dtype=torch.bfloat16, tp_group=None, latent_mode="hidden",
                 engine_config=None):
        self._init_runtime(spec, device, dtype, tp_group)
        if dtype not in (torch.bfloat16, torch.float32):
            raise NotImplementedError(f"{spec.model_type}: dtype {dtype} (bf16 or fp32)")
        if latent_mode not in ("auto", "hidden", "kv"):
            raise NotImplementedError(f"{spec.model_type}: latent_mode {latent_mode!r}; latents are the cached rows")
        self.latent_mode = "kv"
        self.n_q = self.n_kv = 1  # the batch's attention atoms are not used
        self.max_positions = max(8192, getattr(getattr(engine_config, "state_manager", None), "max_context", 0))
        self._build_modules(engine_config)
        self._load(weights)
        self._plan_runs()

    # ------------------------------------------------------------------------------------------
    def _build_modules(self, ec):
        spec, H = self.spec, self.spec.hidden_size
        self.unembed_mod = instantiate_unembed(DSUnembedConfig(model_dim=H, vocab_size=spec.vocab_size,
                                                               norm_type="rms", softcap=spec.logit_softcap), ec)
        self.mixers, self.mlps, self.linears = [], [], []
        for e in spec.layers:
            mix = instantiate_mixer(DSMixerConfig(e["mixer"]["type"], H, e["mixer"], spec.norm_eps, self.tp,
                                                  self.dtype), ec)
            mix.bind_positions(self.max_positions, self.device)
            mix.bind_group(self._allreduce)
            self.mixers.append(mix)
        self._build_layers(ec)
        for lins, mix in zip(self.linears, self.mixers):
            if mix.own_output:
                lins.pop("out.w")
            lins.update({k: instantiate_linear(DSLinearConfig(*io), ec) for k, io in mix.extra_linears().items()})

    def _build_layers(self, ec):
        spec, H = self.spec, self.spec.hidden_size
        self.norm_mod = instantiate_input_norm(
            DSInputNormConfig(H, "rms", spec.norm_eps, spec.input_conv_taps, self.dtype), ec)
        for e, mix in zip(spec.layers, self.mixers):
            ff = e["mlp"]["ff"] if e["mlp"] else 0
            assert ff % self.tp == 0, "the feed-forward width must divide the tensor-parallel size"
            ff //= self.tp
            mlp = instantiate_gated_mlp(DSGatedMLPConfig(H, ff, e["mlp"]["act"]), ec) if e["mlp"] else None
            lins = {"in.w": instantiate_linear(DSLinearConfig(H, mix.in_width), ec),
                    "out.w": instantiate_linear(DSLinearConfig(mix.out_width + ff, H), ec)}
            if mlp is not None:
                lins["up.w"] = instantiate_linear(DSLinearConfig(H, 2 * ff), ec)
            self.mlps.append((mlp, ff))
            self.linears.append(lins)

    def _transform(self, L):
        for k, mod in self.linears[len(self.layers)].items():
            L.w[k] = mod.transform_param(L.w[k])

    def _f32(self, x):
        return None if x is None else x.to(device=self.device, dtype=torch.float32).contiguous()

    def _load(self, sd):
        if sd.get("__presharded__"):
            return self._load_presharded(sd)
        t, f, r = self._t, self._f32, self.tp_rank
        self.embed, self.final_w = t(sd["embed"]), f(sd["final.w"].reshape(-1))
        self.pos_embed = self.lm_head_b = None
        self.final_b = f(sd.get("final.b"))
        self._load_tables(sd)
        lm = sd["lm_head.w"]
        self.vocab = lm.shape[0]
        vs = -(-self.vocab // self.tp)
        shard = lm[r * vs:(r + 1) * vs]
        if shard.shape[0] < vs:  # equal row counts on every rank; the padding columns are cut at ``vocab``
            shard = torch.cat([shard, shard.new_zeros(vs - shard.shape[0], shard.shape[1])])
        self.lm_head = self.embed if shard is sd["embed"] or shard.data_ptr() == sd["embed"].data_ptr() and \
            shard.shape == sd["embed"].shape else t(shard)
        self.layers = []
        for i, Ls in enumerate(sd["layers"]):
            L = _Layer()
            mw = self.mixers[i].shard(Ls["mix"], self._rows, self._cols)
            o = mw.pop("o.w", None)
            self._put(L, mw)
            for k in (f"ln{n}.{kind}" for n in ("1", "2", "1b", "2b") for kind in "wb"):
                if Ls.get(k) is not None:
                    L.w[k] = f(Ls[k].reshape(-1))
            o = self._load_layer(i, L, Ls, o)
            if o is not None:
                L.w["out.w"] = t(o)
            self._transform(L)
            self.layers.append(L)

    def _load_tables(self, sd):
        """Tables by token besides the embedding."""
        self.pair_embed, self.side_embed = self._t(sd.get("pair_embed")), self._t(sd.get("side_embed"))

    def _put(self, L, weights):
        for k, v in weights.items():
            L.w[k] = self._t(v) if v is None or k in _MATRICES or v.dtype != torch.float32 else self._f32(v)

    def _load_layer(self, i, L, Ls, o):
        """The layer's other weights; returns the output projection (the mixer's ``o`` with what joins it)."""
        for k in ("1", "2"):
            cw = Ls.get(f"conv{k}.w")
            L.w[f"conv{k}.w"] = None if cw is None else self._f32(cw.t())  # [taps, W]
        if self.mlps[i][0] is None:
            return o
        L.w["up.w"] = self._t(torch.cat([self._rows(Ls["gate.w"]), self._rows(Ls["up.w"])]))
        return torch.cat([o, self._cols(Ls["down.w"])], 1)

    def _load_presharded(self, sd):
        t, f = self._t, self._f32
        self.embed, self.final_w, self.lm_head = t(sd["embed"]), f(sd["final.w"]), t(sd["lm_head.w"])
        self.pos_embed = self.lm_head_b = None
        self.final_b = f(sd.get("final.b"))
        self._load_tables(sd)
        self.vocab = self.spec.vocab_size
        self.layers = []
        for Ls in sd["layers"]:
            L = _Layer()
            for k, v in Ls.items():
                if isinstance(v, dict):
                    L.w[k] = _PackedWeight(v["q"].to(self.device), v["scales"].to(self.device),
                                           *[int(i) for i in v["meta"]])
                else:
                    self._put(L, {k: v})
            self._transform(L)
            self.layers.append(L)

    def _plan_runs(self):
        self.runs, off = [], 4 if self.spec.pair_embed else 0  # the last token, ahead of the layers' states
        self.row_widths = []
        for li in run_order(self.spec):
            mix = self.mixers[li]
            tail, off = off, off + self._norm_state_floats()
            st, off = off, off + mix.state_floats()
            cache = None
            if mix.cache_row:
                cache = len(self.row_widths)
                self.row_widths.append(mix.cache_row)
            self.runs.append(_Run(li, cache, tail, st))
        self._state_floats = off

    def _norm_state_floats(self):
        return self.norm_mod.state_floats()

    # ------------------------------------------------------------------------------------------
    def kv_cache_config(self):
        return dict(num_layers=len(self.row_widths), n_kv_heads=1, head_dim=0, row_widths=self.row_widths)

    def state_floats(self):
        return self._state_floats

    def save_state(self, batch):
        return None if self.state_pool is None else self.state_pool.data.index_select(0, batch.slots.long())

    def load_state(self, batch, snapshot):
        if snapshot is not None:
            self.state_pool.data.index_copy_(0, batch.slots.long(), snapshot)

    def decode_graph_eligible(self, batch, capture_latents):
        return self.dtype == torch.bfloat16 and super().decode_graph_eligible(batch, capture_latents)

    # ------------------------------------------------------------------------------------------
    # the residual stream: a pair that _start makes, every layer run maps to the next one, and _final reads
    def _start(self, batch):
        return None, None

    def _final(self, stream, idx):
        """The output norm of rows ``idx``, as the unembedding reads them."""
        x, delta = stream
        return norm_rows(x, delta, idx, self.final_w, self.spec.norm_eps)

    def _mix(self, run, x, out, batch):
        i = run.layer
        self.mixers[i](x, self.layers[i], self.linears[i], out, batch,
                       None if run.cache is None else self.kv_cache.get_cache(run.cache), self._state(), run.state)

    def _state(self):
        return None if self.state_pool is None else self.state_pool.data

    def _layer(self, run, stream, batch):
        """One layer run: (new residual, this layer's output, to be added by whoever reads the residual next)."""
        i = run.layer
        x, delta = stream
        L, mix, (mlp, ff), lins = self.layers[i], self.mixers[i], self.mlps[i], self.linears[i]
        gains, convs = [L["ln1.w"]], [L["conv1.w"]]
        if mlp is not None:
            gains.append(L["ln2.w"])
            convs.append(L["conv2.w"])
        x, ys = self.norm_mod(x, delta, gains, convs, batch, self._state(), run.tail, embed=self.embed)
        mid = torch.empty(batch.current_tokens, mix.out_width + ff, dtype=self.dtype, device=self.device)
        self._mix(run, ys[0], mid[:, :mix.out_width], batch)
        if mlp is not None:
            mlp(ys[1], L["up.w"], lins["up.w"], mid[:, mix.out_width:])
        return x, self._allreduce(lins["out.w"](mid, L["out.w"]))

    @torch.no_grad()
    def forward(self, batch, capture_latents=True, sync_latents=True, sink=None):
        """Logits of the wanted rows and the latents ([1, T, W] on the host, or None); see the base class."""
        T = batch.current_tokens
        batch.carry.clear()
        stream = self._start(batch)
        for run in self.runs:
            stream = self._layer(run, stream, batch)
        idx = batch.last_token_idx
        if idx.numel():
            logits = self.unembed_mod.project(self._final(stream, idx), self.lm_head, None, self.tp_group, self.vocab)
        else:
            logits = torch.empty(0, self.vocab, dtype=self.dtype, device=self.device)
        lat, events = None, []
        if capture_latents:
            rows = torch.empty(T, self.latent_width(), dtype=self.dtype, device=self.device)
            self._each_cache(lambda c, r: copy_rows(c, r, batch.tok_seq, batch.tok_pos, batch.block_tables), rows)
            if sink is not None:
                sink(0, rows)
            elif self.latent_width() == 0:
                lat = torch.empty(1, T, 0, dtype=self.dtype)
            else:
                lat = self._latent_buffer(1, T)
                self._d2h(rows, lat[0], events)
        self.latent_event = events[-1] if events else None
        if events and sync_latents:
            events[-1].synchronize()
        return logits, lat

    def _each_cache(self, fn, rows):
        o = 0
        for c, w in enumerate(self.row_widths):
            fn(self.kv_cache.get_cache(c), rows[:, o:o + w])
            o += w

    def latent_layers(self):
        return 1

    def latent_width(self):
        return sum(self.row_widths)

    @torch.no_grad()
    def restore_kv(self, batch, latents):
        """Scatter the sequences' cached rows (host latents, [1, n, W] pieces in batch order) back into their pages."""
        pieces = list(latents) if isinstance(latents, (list, tuple)) else [latents]
        assert sum(p.shape[1] for p in pieces) == batch.current_tokens, "latents must cover exactly the batch's tokens"
        rows = torch.cat([p[0].to(self.device, non_blocking=True) for p in pieces])
        self._each_cache(lambda c, r: copy_rows(c, r, batch.tok_seq, batch.tok_pos, batch.block_tables,
                                                to_cache=True), rows)


class PostNormTransformer(HybridTransformer):
    """Layers with the norm on their sublayers' outputs and routed experts: x += n1(mixer(x)), x += n2(experts(x))."""
    KERNEL_SOURCES = ("act.hip", "experts.hip", "gemv.hip", "grouped_gemm.hip", "output_norm.hip", "paged_attn.hip",
                      "paged_rows.hip")

    def _build_layers(self, ec):
        spec, H = self.spec, self.spec.hidden_size
        self.norm_mod = instantiate_output_norm(DSNormConfig(H, "rms", spec.norm_eps, torch.float32, self.dtype), ec)
        for e, mix in zip(spec.layers, self.mixers):
            m = e["mlp"]
            self.mlps.append(None if m is None else instantiate_expert_layer(
                DSExpertLayerConfig(H, m["ff"], RouterShape(**m["router"]), m["shared_ff"], self.tp, self.dtype), ec))
            self.linears.append({"in.w": instantiate_linear(DSLinearConfig(H, mix.in_width), ec),
                                 "out.w": instantiate_linear(DSLinearConfig(mix.out_width, H), ec)})

    def _load_layer(self, i, L, Ls, o):
        if self.mlps[i] is not None:
            self._put(L, self.mlps[i].shard(Ls["experts"], self._rows, self._cols))
        return o

    def _norm_state_floats(self):
        return 0

    # the stream: (32-bit residual, the rows a sublayer reads)
    def _start(self, batch):
        return self.norm_mod.start(self.embed, batch.input_ids, self.spec.embed_scale)

    def _final(self, stream, idx):
        if not hasattr(self, "_final_gain"):
            self._final_gain = self.final_w * self.spec.logit_scale
        return norm_rows(stream[0], None, idx, self._final_gain, self.spec.norm_eps, self.dtype)

    def _layer(self, run, stream, batch):
        i = run.layer
        L, mix, moe = self.layers[i], self.mixers[i], self.mlps[i]
        x, rows = stream
        mid = torch.empty(batch.current_tokens, mix.out_width, dtype=self.dtype, device=self.device)
        self._mix(run, rows[:, :x.shape[1]], mid, batch)
        x, rows = self.norm_mod(x, self._allreduce(self.linears[i]["out.w"](mid, L["out.w"])), L["ln1.w"])
        if moe is None:
            return x, rows
        parts = moe(rows, L, self.tp_rank)
        if self.tp > 1:
            parts = self._allreduce(moe.total(x, parts))
        return self.norm_mod(x, parts, L["ln2.w"])


class SandwichTransformer(HybridTransformer):
    """Layers with a norm on both sides of every sublayer: x += n1b(mixer(n1(x))), x += n2b(ff(n2(x))); a factor of the
    residual sum is part of the gains of n1b and n2b. With ``token_side``, behind it x += n(proj(gelu(gate x) * e)), e the
    token's row of this layer."""
    KERNEL_SOURCES = ("act.hip", "delta_rule.hip", "gemv.hip", "latent_attn.hip", "output_norm.hip", "paged_attn.hip",
                      "paged_rows.hip")

    def _build_layers(self, ec):
        spec, H = self.spec, self.spec.hidden_size
        self.norm_mod = instantiate_sandwich_norm(
            DSNormConfig(H, "layer" if spec.norm == "ln" else "rms", spec.norm_eps, torch.float32, self.dtype), ec)
        for e, mix in zip(spec.layers, self.mixers):
            m = e["mlp"]
            lins = {"in.w": instantiate_linear(DSLinearConfig(H, mix.in_width), ec),
                    "out.w": instantiate_linear(DSLinearConfig(mix.out_width, H), ec)}
            mlp, ff = None, 0
            if m is not None and m.get("kind") == "moe":
                mlp = instantiate_expert_layer(
                    DSExpertLayerConfig(H, m["ff"], RouterShape(**m["router"]), m.get("shared_ff", 0), self.tp, self.dtype,
                                        m["act"], m.get("limit", 0.0)), ec)
            elif m is not None:
                assert m["ff"] % self.tp == 0, "the feed-forward width must divide the tensor-parallel size"
                ff = m["ff"] // self.tp
                mlp = instantiate_gated_mlp(DSGatedMLPConfig(H, ff, m["act"], m.get("limit", 0.0)), ec)
                lins["up.w"] = instantiate_linear(DSLinearConfig(H, 2 * ff), ec)
                lins["down.w"] = instantiate_linear(DSLinearConfig(ff, H), ec)
            if spec.token_side:
                lins["side.gate.w"] = instantiate_linear(DSLinearConfig(H, spec.token_side), ec)
                lins["side.proj.w"] = instantiate_linear(DSLinearConfig(spec.token_side, H), ec)
            self.mlps.append((mlp, ff))
            self.linears.append(lins)

    def _load_layer(self, i, L, Ls, o):
        mlp, ff = self.mlps[i]
        if "experts" in Ls:
            self._put(L, mlp.shard(Ls["experts"], self._rows, self._cols))
        elif mlp is not None:
            L.w["up.w"] = self._t(torch.cat([self._rows(Ls["gate.w"]), self._rows(Ls["up.w"])]))
            L.w["down.w"] = self._t(self._cols(Ls["down.w"]))
        if self.spec.token_side:
            L.w["side.gate.w"], L.w["side.proj.w"] = self._t(Ls["side.gate.w"]), self._t(Ls["side.proj.w"])
            L.w["side.norm.w"] = self._f32(Ls["side.norm.w"])
        return o

    def _norm_state_floats(self):
        return 0

    # the stream: (32-bit residual or None at the start, the last sublayer's output, its norm)
    def _start(self, batch):
        spec = self.spec
        self._rows_in = (self.embed, batch.input_ids, spec.embed_scale)
        if not spec.pair_embed:
            return None, None, None
        return embed_pairs(self.embed, self.pair_embed, batch.input_ids, spec.embed_scale, spec.pair_embed["mul_prev"],
                           spec.pair_embed["mul_cur"], self._state(), 0, batch), None, None

    def _final(self, stream, idx):
        norm = self.final_w if self.final_b is None else (self.final_w, self.final_b)
        return self.norm_mod(*stream, norm, embed=self._rows_in, idx=idx)[1]

    @staticmethod
    def _norm_of(L, k):
        w, b = L[f"ln{k}.w"], L[f"ln{k}.b"]
        return w if b is None else (w, b)

    def _layer(self, run, stream, batch):
        i = run.layer
        L, mix, (mlp, ff), lins = self.layers[i], self.mixers[i], self.mlps[i], self.linears[i]
        T = batch.current_tokens
        x, rows = self.norm_mod(*stream, self._norm_of(L, "1"), embed=self._rows_in)
        mid = torch.empty(T, mix.out_width, dtype=self.dtype, device=self.device)
        self._mix(run, rows, mid, batch)
        y, norm = mix.output(mid, L, lins, self._allreduce), self._norm_of(L, "1b")
        if mlp is not None:
            if ff:
                x, rows = self.norm_mod(x, y, norm, self._norm_of(L, "2"))
                h = torch.empty(T, ff, dtype=self.dtype, device=self.device)
                mlp(rows, L["up.w"], lins["up.w"], h)
                y = self._allreduce(lins["down.w"](h, L["down.w"]))
            else:
                x, rows = self.norm_mod(x, y, norm, self._norm_of(L, "2"), pad=mlp.row_pad())
                y = mlp(rows, L, self.tp_rank)
                if self.tp > 1:
                    y = self._allreduce(mlp.total(x, y))
            norm = self._norm_of(L, "2b")
        if self.spec.token_side:
            x, rows = self.norm_mod(x, y, norm, None)
            y, norm = self._side(i, rows, batch), L["side.norm.w"]
        return x, y, norm

    def _side(self, i, rows, batch):
        """The layer's own input of every token, gated by the residual."""
        L, lins, n = self.layers[i], self.linears[i], self.spec.token_side
        gate, w, e = lins["side.gate.w"], L["side.gate.w"], self.side_embed[:, i * n:(i + 1) * n]
        g = gather_gemv(rows, w, "gelu_tanh", e, batch.input_ids) if isinstance(gate, BlasFPLinear) else None
        if g is None:
            g = act_gather(gate(rows, w), "gelu_tanh", e, batch.input_ids)
        return lins["side.proj.w"](g, L["side.proj.w"])


class MemorySandwichTransformer(SandwichTransformer):
    """The same layers on layer norms, with matrix memories and parallel mixers (the kernels it runs on are others)."""
    KERNEL_SOURCES = ("act.hip", "experts.hip", "gemv.hip", "grouped_gemm.hip", "head_prep.hip", "matrix_memory.hip",
                      "output_norm.hip", "paged_attn.hip", "paged_rows.hip")
