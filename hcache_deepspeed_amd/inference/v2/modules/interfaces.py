"""Module interfaces + their registries (reference inference/v2/modules/interfaces/*.py)."""
from .module_registry import DSModuleBase, DSModuleRegistryBase


class DSSelfAttentionBase(DSModuleBase):
    """forward(qkv [T, nq + 2 nkv, D] (consumed: RoPE in place), kv_cache (one layer), batch, cos, sin)
    -> attention output [T, nq * D]."""


class DSLinearBase(DSModuleBase):
    """forward(x [T, in], weight (after transform_param), bias=None) -> activation(x W^T + b) [T, out or out/2]."""


class DSMoEBase(DSModuleBase):
    """forward(x [T, H], router_w [E, H], w13 [E, 2I, H], w2 [E, H, I]) -> [T, H] (top-k, dropless)."""


class DSPreNormBase(DSModuleBase):
    """forward(residual, hidden_in, gamma, beta) -> (new residual, normed); hidden_in None: norm(residual)."""


class DSPostNormBase(DSModuleBase):
    """forward(residual, hidden_in, gamma, beta) -> norm(residual + hidden_in)."""


class DSEmbeddingBase(DSModuleBase):
    """forward(batch, word_embeddings, position_embeddings=None) -> [T, H]."""


class DSUnembedBase(DSModuleBase):
    """forward(hidden, residual, batch, lm_head, lm_head_b, final_w, final_b) -> logits of each sequence's last
    token [n_seqs, V_local]."""


class DSInputNormBase(DSModuleBase):
    """forward(x32, delta, gains, convs, batch, state, offset, embed) -> (new 32-bit residual, [one row matrix per
    gain]); ``state_floats()`` per sequence."""


class DSMixerBase(DSModuleBase):
    """Token mixer of one layer. ``in_width`` / ``out_width`` (this rank's); ``cache_row``: values a token stores in
    the paged cache; ``state_floats()``: unpaged float32 state per sequence; ``shard(weights, rows, cols)`` -> this
    rank's weights, with the input projection "in.w" and the output projection "o.w"; ``extra_linears()``: further
    products, name -> (in, out); forward(x, weights, lins, out, batch, cache, state, offset) fills ``out`` [T, out_width],
    ``lins`` holds the linear modules by weight name, ``batch.carry`` what layers of a step hand to later ones.
    ``bind_positions(n, device)``: tables for n positions; ``output(mid, weights, lins, reduce)``: what the layer's norm reads
    (``reduce`` sums a product over the tensor-parallel group). A mixer of its own products (``own_output``) has no "o.w".
    ``bind_group(reduce)``: the same sum, for what a mixer adds up over the group inside."""
    cache_row = 0
    own_output = False

    def state_floats(self):
        return 0

    def extra_linears(self):
        return {}

    def bind_positions(self, positions, device):
        pass

    def bind_group(self, reduce):
        pass

    def output(self, mid, w, lins, reduce):
        return reduce(lins["out.w"](mid, w["out.w"]))


class DSOutputNormBase(DSModuleBase):
    """forward(x32, delta, gain) -> (x32 + gain * norm(delta), the rows the next sublayer reads); delta: a matrix or the
    parts an expert layer returns. ``start(embed, ids, scale)`` -> the same pair for the step's tokens."""


class DSSandwichNormBase(DSModuleBase):
    """forward(x32, delta, norm, next_norm, embed, idx, pad) -> (x32 + norm(delta), next_norm(of that)); a norm is a gain, or
    (gain, bias) of a layer norm; x32 None: the stream starts from ``embed`` (table, ids, scale); ``idx``: the second result
    of these rows only; ``pad``: its rows zero-padded to a multiple of this."""


class DSExpertLayerBase(DSModuleBase):
    """forward(x, weights, rank) -> the output in parts for DSOutputNormBase; ``shard(weights, rows, cols)`` -> this
    rank's weights."""


class DSGatedMLPBase(DSModuleBase):
    """forward(x [T, in], w [gate; up], lin, out [T, I])."""


def _registry(base):

    class _R(DSModuleRegistryBase):
        registry = {}

        @staticmethod
        def associated_class():
            return base

    _R.__name__ = base.__name__.replace("Base", "Registry")
    return _R


DSSelfAttentionRegistry = _registry(DSSelfAttentionBase)
DSLinearRegistry = _registry(DSLinearBase)
DSMoERegistry = _registry(DSMoEBase)
DSPreNormRegistry = _registry(DSPreNormBase)
DSPostNormRegistry = _registry(DSPostNormBase)
DSEmbeddingRegistry = _registry(DSEmbeddingBase)
DSUnembedRegistry = _registry(DSUnembedBase)
DSInputNormRegistry = _registry(DSInputNormBase)
DSMixerRegistry = _registry(DSMixerBase)
DSGatedMLPRegistry = _registry(DSGatedMLPBase)
DSOutputNormRegistry = _registry(DSOutputNormBase)
DSSandwichNormRegistry = _registry(DSSandwichNormBase)
DSExpertLayerRegistry = _registry(DSExpertLayerBase)
