"""The Zikupel decoder as a ``ModelSpec``.

Layers with a norm behind each sublayer and none before, on a float32 stream: ``x += norm1(mixer(x));
x += norm2(ff(x))`` (``parts/block.py: sandwich_norm`` without its first norms), all RMS norms that store
their gain as its distance from one.  A layer's mixer is one of
* ``attention``: grouped-query attention whose values are the keys as projected (biases on q and k, no
  value matrix), an RMS norm of every query and key head before the rotation (half layout, on the first
  ``rot.dims`` elements, YaRN frequencies), softly capped scores, and the heads' results times
  ``sigmoid(W_g x)`` before the output product (options of ``parts/attention.py``);
* ``lightning``: a matrix state with a fixed decay per head (``parts/linear_attention.py:
  lightning_attention``).
The feed-forward is ``W_down(silu(W_gate x) * W_up x)``, or routed experts without a gate, ``W_down
relu(W_up w x)^2`` with the router's sigmoid w on the expert's input, beside a shared one
(``parts/moe.py``), or absent.  The head is a matrix of its own.  Tensor names: ``embed``,
``final.norm``, ``head``, ``l<i>.{norm1, norm2}``, ``l<i>.mix.{q, k, g, o}`` with ``q.b``, ``k.b``,
``q.norm``, ``k.norm``, or ``l<i>.mix.{q, k, v, g, o, norm}``, ``l<i>.mlp.{gate, up, down}`` or
``l<i>.mlp.{router, e<k>.up, e<k>.down, shared.up, shared.down}``.
"""

from __future__ import annotations

from kvcore_amd.config.zikupel_config import DenseConfig, KeyValueAttentionConfig, SquaredExpertsConfig, ZikupelConfig
from kvcore_amd.parts.base import PartSpec

from .spec import LayerSpec, ModelSpec


def zikupel_spec(config: ZikupelConfig) -> ModelSpec:
    H, eps = config.width, config.eps

    def norm() -> PartSpec:
        return PartSpec("rmsnorm", {"hidden_size": H, "eps": eps, "weight_offset": 1.0, "weight_name": ""})

    positions: list[PartSpec] = []
    position_index: dict[tuple, int] = {}

    def rotation(m: KeyValueAttentionConfig) -> int | None:
        """The index of the rotary encoding with this layer's constants among ``positions``."""
        if m.rot_dims <= 0:
            return None
        key = (m.rot_dims, m.rot_base, m.yarn)
        if key not in position_index:
            position_index[key] = len(positions)
            positions.append(PartSpec("rotary", {"rot_dim": m.rot_dims, "theta": m.rot_base,
                                                 "scaling": None if m.yarn is None else m.yarn.as_scaling()}))
        return position_index[key]

    layers: list[LayerSpec] = []
    unread: list[str] = []  # the norm of a second sublayer that a layer without a feed-forward may still carry
    for i, layer in enumerate(config.layers):
        m = layer.mixer
        position = None
        if isinstance(m, KeyValueAttentionConfig):
            position = rotation(m)
            mixer = PartSpec("paged_attention", {
                "hidden_size": H, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim,
                "scale": m.scale, "softcap": m.softcap, "bias": True, "o_bias": False, "qk_norm_eps": eps,
                "values_are_keys": True, "output_gate": True, "float32_result": True, "sized_buffers": True,
                "tensor_names": {"q": "q", "k": "k", "g": "g", "o": "o", "q_bias": "q.b", "k_bias": "k.b",
                                 "q_norm": "q.norm", "k_norm": "k.norm"}})
        else:
            mixer = PartSpec("lightning_attention", {
                "hidden_size": H, "heads": m.heads, "dim": m.dim, "vdim": m.vdim, "decay": m.decay, "eps": eps,
                "float32_result": True,
                "tensor_names": {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "norm": "norm"}})
        norms = {name: norm() for name in ("norm1", "norm2")}
        if layer.mlp is None:
            ffn = PartSpec("none")
            del norms["norm2"]
            unread.append(f"l{i}.norm2")
        elif isinstance(layer.mlp, DenseConfig):
            ffn = PartSpec("swiglu", {
                "hidden_size": H, "intermediate_size": layer.mlp.ff, "gate_name": "gate", "up_name": "up",
                "down_name": "down", "suffix": "", "sized_buffers": True, "float32_result": True})
        else:
            assert isinstance(layer.mlp, SquaredExpertsConfig)
            e = layer.mlp
            ffn = PartSpec("routed_experts", {
                "hidden_size": H, "experts": e.experts, "top": e.top, "expert_size": e.ff, "limit": None,
                "score": "sigmoid", "renormalize": False, "weight_on_input": True, "activation": "relu_squared",
                "shared_size": e.shared_ff,
                "tensor_names": {"router": "router", "expert": "e{e}", "shared": "shared", "up": "up",
                                 "down": "down"}})
        layers.append(LayerSpec(
            prefix=f"l{i}", mixer=mixer, ffn=ffn, norms=norms, position=position,
            block=PartSpec("sandwich_norm", {"mixer_name": "mix", "ffn_name": "mlp", "pre_mixer": None,
                                             "post_mixer": "norm1", "pre_ffn": None, "post_ffn": "norm2"})))

    return ModelSpec(
        vocab_size=config.vocab, hidden_size=H, max_position_embeddings=config.max_position_embeddings,
        layers=tuple(layers), final_norm=norm(), positions=tuple(positions),
        embedding=PartSpec("token_embedding", {"vocab_size": config.vocab, "hidden_size": H, "weight_name": "embed"}),
        head=PartSpec("linear_head", {"vocab_size": config.vocab, "hidden_size": H, "weight_name": ""}),
        tie_word_embeddings=False, eos_token_ids=config.eos_token_ids, embed_prefix="",
        final_norm_prefix="final.norm", head_prefix="head", ignored_suffixes=tuple(unread),
    )
