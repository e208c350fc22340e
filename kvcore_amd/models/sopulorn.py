"""The Sopulorn decoder as a ``ModelSpec``.

A token's row plus the row of its pair with the token before (``parts/embedding.py:
pair_embedding``), then layers with a norm before and a norm behind each sublayer on a float32
stream (``parts/block.py: sandwich_norm``), all RMS norms that store their gain as its distance
from one.  The mixer is grouped-query attention with biases on q, k and v, an RMS norm of every
query and key head before the rotation (half layout, on the first ``rot.dims`` elements) and a sink
of score zero in the softmax's denominator (options of ``parts/attention.py``); a layer with
``kv_from`` has queries alone and reads the cache of the layer it names.  The feed-forward is
gated and clamped, ``W_down(g sigmoid(GLU_ALPHA g) (u + 1))`` (``parts/mlp.py``), or routed experts
weighted by a softmax over the chosen logits beside a shared expert with a gate a token
(``parts/moe.py``), or absent.  The head is a matrix of its own.  Tensor names: ``embed``,
``bigram``, ``final.norm``, ``head``, ``l<i>.{norm1, norm1b, norm2, norm2b}``,
``l<i>.mix.{q, k, v, o}`` with ``q.b``, ``k.b``, ``v.b``, ``q.norm``, ``k.norm``,
``l<i>.mlp.{gate, up, down}`` or ``l<i>.mlp.{router, router.b, e<k>.*, shared.*, shared.sg}``.
"""

from __future__ import annotations

from kvcore_amd.config.sopulorn_config import ClampedFeedForwardConfig, GatedExpertsConfig, SopulornConfig
from kvcore_amd.parts.base import PartSpec

from .spec import LayerSpec, ModelSpec, ScheduleEntry

GLU_ALPHA = 1.702   # the dense feed-forward's activation: g * sigmoid(GLU_ALPHA * g) * (u + UP_SHIFT)
UP_SHIFT = 1.0
SINK_SCORE = 0.0    # of the term in the softmax's denominator that has no key


def sopulorn_spec(config: SopulornConfig) -> ModelSpec:
    H, eps = config.width, config.eps

    def norm() -> PartSpec:
        return PartSpec("rmsnorm", {"hidden_size": H, "eps": eps, "weight_offset": 1.0, "weight_name": ""})

    positions: list[PartSpec] = []
    position_index: dict[tuple, int] = {}

    def rotation(dims: int, base: float) -> int | None:
        """The index of the rotary encoding with these constants among ``positions``."""
        if dims <= 0:
            return None
        if (dims, base) not in position_index:
            position_index[dims, base] = len(positions)
            positions.append(PartSpec("rotary", {"rot_dim": dims, "theta": base}))
        return position_index[dims, base]

    layers: list[LayerSpec] = []
    unread: list[str] = []  # norms of a second sublayer that a layer without a feed-forward may still carry
    for i, layer in enumerate(config.layers):
        m = layer.mixer
        mixer = PartSpec("paged_attention", {
            "hidden_size": H, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim,
            "v_head_dim": m.vdim, "scale": m.scale, "bias": True, "o_bias": False, "qk_norm_eps": eps,
            "sinks": SINK_SCORE, "own_kv": m.kv_from is None, "float32_result": True, "sized_buffers": True,
            "tensor_names": {"q": "q", "k": "k", "v": "v", "o": "o", "q_bias": "q.b", "k_bias": "k.b",
                             "v_bias": "v.b", "q_norm": "q.norm", "k_norm": "k.norm"}})
        norms = {name: norm() for name in ("norm1", "norm1b", "norm2", "norm2b")}
        if layer.mlp is None:
            ffn = PartSpec("none")
            for name in ("norm2", "norm2b"):
                del norms[name]
                unread.append(f"l{i}.{name}")
        elif isinstance(layer.mlp, ClampedFeedForwardConfig):
            ffn = PartSpec("swiglu", {
                "hidden_size": H, "intermediate_size": layer.mlp.ff, "gate_name": "gate", "up_name": "up",
                "down_name": "down", "suffix": "", "sized_buffers": True, "activation": "clamped",
                "limit": layer.mlp.limit, "alpha": GLU_ALPHA, "up_shift": UP_SHIFT, "float32_result": True})
        else:
            assert isinstance(layer.mlp, GatedExpertsConfig)
            e = layer.mlp
            ffn = PartSpec("routed_experts", {
                "hidden_size": H, "experts": e.experts, "top": e.top, "expert_size": e.ff, "limit": None,
                "alpha": 1.0, "up_shift": 0.0, "score": "logit", "router_bias": True,
                "shared_size": e.shared_ff, "shared_gate": e.shared_ff > 0,
                "tensor_names": {"router": "router", "router_bias": "router.b", "expert": "e{e}", "shared": "shared",
                                 "shared_gate": "shared.sg", "gate": "gate", "up": "up", "down": "down"}})
        layers.append(LayerSpec(
            prefix=f"l{i}", mixer=mixer, ffn=ffn, norms=norms, position=rotation(m.rot_dims, m.rot_base),
            block=PartSpec("sandwich_norm", {"mixer_name": "mix", "ffn_name": "mlp"})))

    table = {"vocab_size": config.vocab, "hidden_size": H, "weight_name": "embed"}
    if config.bigram is None:
        embedding = PartSpec("token_embedding", table)
    else:
        b = config.bigram
        embedding = PartSpec("pair_embedding", {**table, "pairs_name": "bigram", "buckets": b.buckets,
                                                "mul_prev": b.mul_prev, "mul_cur": b.mul_cur})
    return ModelSpec(
        vocab_size=config.vocab, hidden_size=H, max_position_embeddings=config.max_position_embeddings,
        layers=tuple(layers), final_norm=norm(), positions=tuple(positions),
        schedule=tuple(ScheduleEntry(i, cache_from=layer.mixer.kv_from) for i, layer in enumerate(config.layers)),
        embedding=embedding,
        head=PartSpec("linear_head", {"vocab_size": config.vocab, "hidden_size": H, "weight_name": ""}),
        tie_word_embeddings=False, eos_token_ids=config.eos_token_ids, embed_prefix="",
        final_norm_prefix="final.norm", head_prefix="head", ignored_suffixes=tuple(unread),
    )
