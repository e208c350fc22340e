"""Sopulorn without a GPU: configuration, registry, the schedule of borrowed caches, the checkpoint
layout, caches and states as the model plans them, and the plain implementation's own consistency."""

from __future__ import annotations

import copy
import math
import random

import pytest
import torch

from tests.plain import sopulorn as plain
from tests.sopulorn_helpers import CONFIG_A, CONFIG_B, CONFIG_C, CONFIG_D, CONFIGS, attn, dense, layer, model, random_config

F = torch.float64


def spec_of(config):
    from kvcore_amd.registry import resolve_architecture

    arch = resolve_architecture(config)
    return arch.build_spec(arch.parse_config(config))


def decoder(config):
    from kvcore_amd.models.decoder import DecoderModel

    return DecoderModel(spec_of(config), torch.float32, "cpu")


def test_the_architecture_is_registered():
    from kvcore_amd.registry import resolve_architecture

    assert resolve_architecture(CONFIG_A).name == "Sopulorn"


def test_borrowing_layers_read_the_plane_their_owner_writes():
    m = decoder(CONFIG_A)
    calls = m.calls
    assert [c.write_cache for c in calls] == [True, True, False, False, True]
    assert (calls[2].group_index, calls[2].cache_index) == (calls[0].group_index, calls[0].cache_index)
    assert (calls[3].group_index, calls[3].cache_index) == (calls[1].group_index, calls[1].cache_index)
    needs = {g.need.planes: g.num_planes for g in m.cache_groups}
    assert needs == {((2, 24), (2, 40)): 1, ((3, 16), (3, 16)): 1, ((2, 16), (2, 24)): 1}
    # layers of equal sizes share a group; readers take no plane
    assert {g.need.planes: g.num_planes for g in decoder(CONFIG_D).cache_groups}[((1, 32), (1, 16))] == 1
    # values of twice the keys' size lie in two planes
    assert any(g.need.planes == ((1, 64), (1, 64), (1, 64)) for g in decoder(CONFIG_B).cache_groups)


def test_the_embedding_s_state_is_one_token_a_slot():
    m = decoder(CONFIG_A)
    assert m.embed_states == (0,) and m.state_arrays[0].need.shape == (1,)
    assert m.state_arrays[0].need.dtype == torch.int32
    assert decoder(CONFIG_D).state_arrays == [] and decoder(CONFIG_D).embed_states == ()


def test_checkpoint_layout_has_the_design_s_names_and_shapes():
    from kvcore_amd.weights.loader import checkpoint_layout

    layout = {k: v[0] for k, v in checkpoint_layout(spec_of(CONFIG_A)).items()}
    assert layout["embed"] == (211, 96) and layout["bigram"] == (102, 96) and layout["head"] == (211, 96)
    assert layout["final.norm"] == (96,)
    assert layout["l0.mix.q"] == (96, 96) and layout["l0.mix.k"] == (48, 96) and layout["l0.mix.v"] == (80, 96)
    assert layout["l0.mix.q.b"] == (96,) and layout["l0.mix.v.b"] == (80,) and layout["l0.mix.o"] == (96, 160)
    assert layout["l0.mix.q.norm"] == (24,) and layout["l0.mix.k.norm"] == (24,)
    assert "l0.mix.o.b" not in layout and "l0.mlp.gate.b" not in layout
    assert layout["l0.mlp.gate"] == (80, 96) and layout["l0.mlp.down"] == (96, 80)
    assert {k for k in layout if k.startswith("l2.mix.")} == {"l2.mix.q", "l2.mix.q.b", "l2.mix.q.norm", "l2.mix.o"}
    assert layout["l1.mlp.router"] == (12, 96) and layout["l1.mlp.router.b"] == (12,)
    assert layout["l1.mlp.e11.gate"] == (24, 96) and layout["l1.mlp.shared.down"] == (96, 40)
    assert layout["l1.mlp.shared.sg"] == (1, 96) and not any(".shared" in k for k in layout if k.startswith("l2."))
    assert all(f"l0.norm{x}" in layout for x in ("1", "1b", "2", "2b"))
    assert "l3.norm2" not in layout and "l3.norm2b" not in layout and "l3.norm1b" in layout
    assert "bigram" not in checkpoint_layout(spec_of(CONFIG_D))


def test_wrong_configurations_are_refused_by_name():
    from kvcore_amd.config.model_config import ConfigError

    def broken(change):
        config = copy.deepcopy(CONFIG_A)
        change(config)
        with pytest.raises(ConfigError) as info:
            spec_of(config)
        return str(info.value)

    assert "kv_heads" in broken(lambda c: c["layers"][0]["mixer"].update(kv_heads=3))
    assert "rot.dims" in broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=26))
    assert "rot.dims" in broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=3))
    assert "scale" in broken(lambda c: c["layers"][0]["mixer"].pop("scale"))
    assert "kv_from" in broken(lambda c: c["layers"][2]["mixer"].update(kv_from=2))   # itself
    assert "kv_from" in broken(lambda c: c["layers"][3]["mixer"].update(kv_from=2))   # a layer that borrows
    assert "kv_from" in broken(lambda c: c["layers"][2]["mixer"].update(kv_from=1))   # other sizes
    assert "type" in broken(lambda c: c["layers"][0].update(type="mamba"))
    assert "kind" in broken(lambda c: c["layers"][0]["mlp"].update(kind="glu"))
    assert "limit" in broken(lambda c: c["layers"][0]["mlp"].pop("limit"))
    assert "experts" in broken(lambda c: c["layers"][1]["mlp"]["router"].update(top=13))
    assert "shared" in broken(lambda c: c["layers"][1]["mlp"]["shared"].update(ff=0))
    assert "bigram" in broken(lambda c: c["embedding"]["bigram"].update(buckets=0))
    assert "mul_cur" in broken(lambda c: c["embedding"]["bigram"].pop("mul_cur"))


def test_every_drawn_configuration_builds():
    for seed in range(40):
        config = random_config(random.Random(seed))
        m = decoder(config)
        assert len(m.calls) == len(config["layers"])
        assert [c.write_cache for c in m.calls] == [l["mixer"].get("kv_from") is None for l in config["layers"]]


def _weights(config, seed=0, std=0.3):
    from kvcore_amd.weights.loader import checkpoint_layout

    gen = torch.Generator().manual_seed(seed)
    return {name: torch.randn(shape, generator=gen, dtype=F) * std
            for name, (shape, _, _) in checkpoint_layout(spec_of(config)).items()}


def test_plain_pair_rows_by_hand():
    b = {"buckets": 10, "mul_prev": 3, "mul_cur": 7}
    assert plain.bigram_rows([4, 5, 0, 9], b) == [10, (12 + 35) % 10, 15 % 10, 63 % 10]
    assert plain.bigram_rows([2**20, 2**20], dict(b, mul_prev=2**20)) == [10, (2**40 + 7 * 2**20) % 10]


def test_plain_softmax_counts_one_more():
    s = torch.tensor([[0.0, 9.0], [math.log(2.0), math.log(3.0)]], dtype=F)
    p = plain.softmax_with_one(s)
    assert torch.allclose(p, torch.tensor([[0.5, 0.0], [2 / 6, 3 / 6]], dtype=F))
    big = plain.softmax_with_one(torch.full((1, 1), -800.0, dtype=F))
    assert float(big) == pytest.approx(0.0, abs=1e-300)


def test_plain_rotation_turns_pairs_half_a_rotated_width_apart():
    x = torch.zeros(3, 1, 6, dtype=F)
    x[:, 0, 0], x[:, 0, 5] = 1.0, 2.0
    y = plain.rotate(x, 4, 100.0)
    assert torch.allclose(y[2, 0, [0, 2]], torch.tensor([math.cos(2.0), math.sin(2.0)], dtype=F))
    assert torch.equal(y[:, 0, 5], x[:, 0, 5]) and torch.equal(y[0], x[0])
    x = torch.zeros(3, 1, 6, dtype=F)
    x[:, 0, 1] = 1.0  # the second pair turns base^(-2/dims) as fast
    assert torch.allclose(plain.rotate(x, 4, 100.0)[2, 0, [1, 3]],
                          torch.tensor([math.cos(0.2), math.sin(0.2)], dtype=F))


def test_plain_routing_by_hand():
    h = torch.eye(3, dtype=F)[:1]
    w = {"router": torch.zeros(4, 3, dtype=F), "router.b": torch.tensor([0.0, 5.0, 0.0, 0.0], dtype=F)}
    w["router"][:, 0] = torch.tensor([3.0, -3.0, 1.0, -1.0], dtype=F)
    choice, weight = plain.route(h, w, {"top": 2})
    assert choice[0].tolist() == [0, 1]  # logits 3, 2, 1, -1 with the bias
    assert float(weight[0, 0]) == pytest.approx(math.e / (math.e + 1))


def test_plain_model_is_causal_and_borrowing_layers_use_their_owner_s_keys():
    config = model(50, 32, 1e-5, (13, 5, 3), [layer(attn(2, 1, 8, 6, 0.5), dense(16, 1.0)),
                                              layer(attn(2, 1, 8, 6, 0.3, kv_from=0), dense(16, 1.0))])
    w = _weights(config)
    a = [3, 7, 1, 9, 4, 4, 8]
    base = plain.forward(config, w, a)
    b = a[:5] + [11] + a[6:]
    moved = plain.forward(config, w, b)
    assert torch.equal(base[:5], moved[:5]) and not torch.allclose(base[5], moved[5])
    stream: list = []
    plain.forward(config, w, a, stream)
    # layer 1 once more by hand, its keys and values made from layer 0's input
    x0 = plain.embedding(config, w, a)
    h0 = plain.offset_norm(x0, w["l0.norm1"], 1e-5)
    kv = plain.keys_and_values(h0, plain.sub(w, "l0.mix."), config["layers"][0]["mixer"], 1e-5)
    h1 = plain.offset_norm(stream[0], w["l1.norm1"], 1e-5)
    y = plain.attention(h1, plain.sub(w, "l1.mix."), config["layers"][1]["mixer"], 1e-5, kv)
    x = stream[0] + plain.offset_norm(y, w["l1.norm1b"], 1e-5)
    f = plain.dense_ff(plain.offset_norm(x, w["l1.norm2"], 1e-5), plain.sub(w, "l1.mlp."), config["layers"][1]["mlp"])
    assert torch.allclose(x + plain.offset_norm(f, w["l1.norm2b"], 1e-5), stream[1], atol=1e-12)


def test_configurations_cover_what_they_say():
    mixers = [l["mixer"] for c, _ in CONFIGS.values() for l in c["layers"]]
    ratios = {m["vdim"] / m["dim"] for m in mixers}
    assert {0.5, 1.0, 2.0} <= ratios and len(ratios) > 5
    assert any("rot" not in m for m in mixers) and any(m["rot"]["dims"] < m["dim"] for m in mixers if "rot" in m)
    assert any(l["mlp"] is None for l in CONFIG_A["layers"]) and "embedding" not in CONFIG_D
    assert CONFIG_C["embedding"]["bigram"]["buckets"] == 1
