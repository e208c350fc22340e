"""Zikupel without a GPU: configuration, registry, the checkpoint layout, caches and states as the model
plans them, the YaRN frequencies, and the plain implementation's own consistency."""

from __future__ import annotations

import copy
import math
import random

import pytest
import torch

from tests.plain import zikupel as plain
from tests.zikupel_helpers import (CONFIG_A, CONFIG_B, CONFIG_C, CONFIG_D, CONFIGS, attn, dense, layer, lightning, model, moe,
                                   random_config, yarn)

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

    assert resolve_architecture(CONFIG_A).name == "Zikupel"


def test_caches_and_states_as_the_model_plans_them():
    m = decoder(CONFIG_A)
    needs = {g.need.planes: g.num_planes for g in m.cache_groups}
    assert needs == {((2, 24), (2, 24)): 1, ((3, 16), (3, 16)): 1, ((1, 40), (1, 40)): 1}
    assert [s.need.shape for s in m.state_arrays] == [(3, 24, 40), (2, 12, 5)]  # rows rounded up to fours
    assert all(s.need.dtype == torch.float32 for s in m.state_arrays)
    assert m.graph_safe()
    # layers of equal sizes share a group
    b = {g.need.planes: g.num_planes for g in decoder(CONFIG_B).cache_groups}
    assert b == {((2, 64), (2, 64)): 3, ((1, 128), (1, 128)): 1, ((8, 64), (8, 64)): 1}
    # layers with equal rotation constants share its tables
    two = model(50, 32, 1e-5, [layer(attn(2, 1, 8, 0.5, 4.0, 4, 100.0, yarn(2.0, 16, 4.0, 1.0)), dense(16))] * 2)
    assert len(decoder(two).positions) == 1 and len(decoder(CONFIG_B).positions) == 4


def test_checkpoint_layout_has_the_design_s_names_and_shapes():
    from kvcore_amd.weights.loader import checkpoint_layout

    layout = {k: v[0] for k, v in checkpoint_layout(spec_of(CONFIG_A)).items()}
    assert layout["embed"] == (211, 96) and layout["head"] == (211, 96) and layout["final.norm"] == (96,)
    assert {k: v for k, v in layout.items() if k.startswith("l0.")} == {
        "l0.norm1": (96,), "l0.norm2": (96,), "l0.mix.q": (96, 96), "l0.mix.q.b": (96,), "l0.mix.k": (48, 96),
        "l0.mix.k.b": (48,), "l0.mix.q.norm": (24,), "l0.mix.k.norm": (24,), "l0.mix.g": (96, 96), "l0.mix.o": (96, 96),
        "l0.mlp.gate": (80, 96), "l0.mlp.up": (80, 96), "l0.mlp.down": (96, 80)}
    assert {k: v for k, v in layout.items() if k.startswith("l1.mix")} == {
        "l1.mix.q": (72, 96), "l1.mix.k": (72, 96), "l1.mix.v": (120, 96), "l1.mix.g": (120, 96), "l1.mix.o": (96, 120),
        "l1.mix.norm": (120,)}
    assert layout["l1.mlp.router"] == (12, 96) and layout["l1.mlp.e11.up"] == (24, 96)
    assert layout["l1.mlp.e0.down"] == (96, 24) and layout["l1.mlp.shared.up"] == (40, 96)
    assert not any(k.endswith("gate") for k in layout if k.startswith("l1.mlp"))
    assert not any("shared" in k for k in layout if k.startswith("l2."))
    assert "l3.norm2" not in layout and "l3.norm1" in layout


def test_the_gate_s_rows_have_no_bias():
    m = decoder(CONFIG_A)
    bias = m.blocks[0].mixer.params["qkv_proj.bias"]
    bias.fill_(3.0)
    m.weights_loaded()
    assert bias.numel() == 96 + 48 + 96 and float(bias[:144].min()) == 3.0 and float(bias[144:].abs().max()) == 0.0


def test_wrong_configurations_are_refused_by_name():
    from kvcore_amd.config.model_config import ConfigError

    def broken(change):
        config = copy.deepcopy(CONFIG_A)
        change(config)
        with pytest.raises(ConfigError) as info:
            spec_of(config)
        return str(info.value)

    assert "kv_heads" in broken(lambda c: c["layers"][0]["mixer"].update(kv_heads=3))
    assert "vdim" in broken(lambda c: c["layers"][0]["mixer"].update(vdim=16))
    assert "rot.dims" in broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=26))
    assert "rot.dims" in broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=3))
    assert "scale" in broken(lambda c: c["layers"][0]["mixer"].pop("scale"))
    assert "softcap" in broken(lambda c: c["layers"][0]["mixer"].update(softcap=-1.0))
    assert "softcap" in broken(lambda c: c["layers"][0]["mixer"].update(softcap=0))
    assert "original" in broken(lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("original"))
    assert "factor" in broken(lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0))
    assert "decay" in broken(lambda c: c["layers"][1]["mixer"].update(decay=[0.5, 0.5]))
    assert "decay" in broken(lambda c: c["layers"][1]["mixer"].pop("decay"))
    assert "vdim" in broken(lambda c: c["layers"][1]["mixer"].update(vdim=0))
    assert "type" in broken(lambda c: c["layers"][0].update(type="mamba"))
    assert "kind" in broken(lambda c: c["layers"][0]["mlp"].update(kind="glu"))
    assert "experts" in broken(lambda c: c["layers"][1]["mlp"]["router"].update(top=13))
    assert "shared" in broken(lambda c: c["layers"][1]["mlp"]["shared"].update(ff=0))


def test_every_drawn_configuration_builds():
    for seed in range(40):
        config = random_config(random.Random(seed))
        m = decoder(config)
        kinds = [l["type"] for l in config["layers"]]
        assert len(m.state_arrays) == kinds.count("lightning")
        assert sum(g.num_planes for g in m.cache_groups) == kinds.count("attention")


@pytest.mark.parametrize("dims,base,scaling", [
    (64, 10000.0, yarn(8.0, 256, 32.0, 1.0)), (16, 500.0, yarn(4.0, 64, 8.0, 1.0)), (32, 1e6, yarn(40.0, 4096, 32.0, 1.0)),
    (2, 10000.0, yarn(2.0, 100, 4.0, 1.0)), (8, 100.0, yarn(3.0, 6, 32.0, 1.0)), (48, 500.0, yarn(2.0, 10 ** 6, 32.0, 1.0)),
    (24, 10000.0, yarn(16.0, 100, 3.0, 3.0)), (32, 10000.0, None)])
def test_yarn_frequencies(dims, base, scaling):
    """The product's table against the plain one, also where the ramp lies outside the pairs on either
    side and where it has no width."""
    from kvcore_amd.parts.rotary import rotary_inv_freq, rotary_table_scale

    given = None if scaling is None else {"rope_type": "yarn", **scaling}
    want, factor = plain.frequencies({"dims": dims, "base": base, "scaling": scaling})
    assert torch.allclose(rotary_inv_freq(dims, base, given).double(), torch.tensor(want, dtype=F), rtol=1e-6, atol=0)
    assert rotary_table_scale(given) == pytest.approx(factor, abs=1e-12)


def test_plain_yarn_by_hand():
    # pairs of 8 elements, base 10^4: the pair that turns t times over 2 pi 100 positions is 4 log10(100 / t) / 4
    rot = {"dims": 8, "base": 1e4, "scaling": yarn(10.0, 2 * math.pi * 100, 100.0, 1.0)}
    freqs, factor = plain.frequencies(rot)
    assert plain.turns_dim(100.0, 8, 1e4, 2 * math.pi * 100) == pytest.approx(0.0, abs=1e-9)
    assert plain.turns_dim(1.0, 8, 1e4, 2 * math.pi * 100) == pytest.approx(2.0)
    assert freqs == pytest.approx([1.0, 0.1 * (0.5 * 0.1 + 0.5), 0.01 / 10, 0.001 / 10])
    assert factor == pytest.approx(0.1 * math.log(10.0) + 1.0)
    assert plain.frequencies({"dims": 4, "base": 100.0}) == ([1.0, 0.1], 1.0)


def test_plain_rotation_turns_pairs_half_a_rotated_width_apart():
    rot = {"dims": 4, "base": 100.0}
    x = torch.zeros(3, 1, 6, dtype=F)
    x[:, 0, 0], x[:, 0, 5] = 1.0, 2.0
    y = plain.rotate(x, rot)
    assert torch.allclose(y[2, 0, [0, 2]], torch.tensor([math.cos(2.0), math.sin(2.0)], dtype=F))
    assert torch.equal(y[:, 0, 5], x[:, 0, 5]) and torch.equal(y[0], x[0])
    scaled = plain.rotate(x, dict(rot, scaling=yarn(math.e ** 10, 10 ** 9, 4.0, 1.0)))  # every pair keeps its frequency
    assert torch.allclose(scaled[:, :, :4], 2.0 * y[:, :, :4]) and torch.equal(scaled[:, 0, 5], x[:, 0, 5])


def test_plain_cap_and_softmax_by_hand():
    assert torch.allclose(plain.capped(torch.tensor([0.0, 1.0, 1e6, -1e6], dtype=F), 5.0),
                          torch.tensor([0.0, 5 * math.tanh(0.2), 5.0, -5.0], dtype=F))
    p = plain.causal_softmax(torch.tensor([[0.0, 9.0], [math.log(1.0), math.log(3.0)]], dtype=F))
    assert torch.allclose(p, torch.tensor([[1.0, 0.0], [0.25, 0.75]], dtype=F))


def test_plain_lightning_state_is_the_decayed_sum():
    gen = torch.Generator().manual_seed(3)
    q, k = (torch.randn(7, 2, 3, generator=gen, dtype=F) for _ in range(2))
    v = torch.randn(7, 2, 4, generator=gen, dtype=F)
    got = plain.lightning_state(q, k, v, [0.7, 1.0])
    for h, lam in enumerate((0.7, 1.0)):
        for t in range(7):
            want = sum(lam ** (t - j) * (k[j, h] @ q[t, h]) * v[j, h] for j in range(t + 1))
            assert torch.allclose(got[t, h], want)
    zero = plain.lightning_state(q, k, v, [0.0, 0.0])  # a state that forgets everything
    assert torch.allclose(zero[4, 1], (k[4, 1] @ q[4, 1]) * v[4, 1])


def test_plain_routing_and_weight_on_the_input_by_hand():
    w = {"router": torch.tensor([[3.0], [-3.0], [1.0], [-1.0]], dtype=F)}
    choice, weight = plain.route(torch.ones(1, 1, dtype=F), w, 2)
    assert choice[0].tolist() == [0, 2]
    assert torch.allclose(weight[0], torch.sigmoid(torch.tensor([3.0, 1.0], dtype=F)))  # they do not sum to one
    gen = torch.Generator().manual_seed(4)
    h = torch.randn(3, 1, generator=gen, dtype=F).abs()
    w.update({f"e{e}.up": torch.randn(5, 1, generator=gen, dtype=F) for e in range(4)})
    w.update({f"e{e}.down": torch.randn(1, 5, generator=gen, dtype=F) for e in range(4)})
    got = plain.routed_ff(h, w, {"router": {"top": 1}})
    s = torch.sigmoid(3.0 * h)
    assert torch.allclose(got, s ** 2 * plain.expert(h, w, "e0"))  # the activation is a square


def test_plain_model_is_causal_and_has_norms_behind_its_sublayers_only():
    from kvcore_amd.weights.loader import checkpoint_layout

    config = model(50, 32, 1e-5, [layer(attn(2, 1, 8, 0.5, 4.0, 4, 100.0), dense(16)),
                                  layer(lightning(6, 10, 0.9, 0.5), moe(8, 4, 2, 12))])
    gen = torch.Generator().manual_seed(0)
    w = {name: torch.randn(shape, generator=gen, dtype=F) * 0.3
         for name, (shape, _, _) in checkpoint_layout(spec_of(config)).items()}
    a = [3, 7, 1, 9, 4, 4, 8]
    base = plain.forward(config, w, a)
    moved = plain.forward(config, w, a[:5] + [11] + a[6:])
    assert torch.equal(base[:5], moved[:5]) and not torch.allclose(base[5], moved[5]) and not torch.allclose(base[6], moved[6])
    stream: list = []
    plain.forward(config, w, a, stream)
    x = w["embed"][torch.tensor(a)]
    m = plain.attention(x, plain.sub(w, "l0.mix."), config["layers"][0]["mixer"], 1e-5)
    x = x + m / torch.sqrt((m * m).mean(1, keepdim=True) + 1e-5) * (1 + w["l0.norm1"])
    f = (plain.silu(x @ w["l0.mlp.gate"].T) * (x @ w["l0.mlp.up"].T)) @ w["l0.mlp.down"].T
    x = x + f / torch.sqrt((f * f).mean(1, keepdim=True) + 1e-5) * (1 + w["l0.norm2"])
    assert torch.allclose(x, stream[0], atol=1e-12)


def test_configurations_cover_what_they_say():
    mixers = [(l["type"], l["mixer"]) for c, _ in CONFIGS.values() for l in c["layers"]]
    caps = {m.get("softcap") for t, m in mixers if t == "attention"}
    assert None in caps and any(c and c > 44 for c in caps) and any(c and c <= 44 for c in caps)
    assert any("rot" not in m for t, m in mixers if t == "attention")
    assert any(m["rot"]["dims"] < m["dim"] for t, m in mixers if "rot" in m)
    assert any("scaling" not in m["rot"] for t, m in mixers if "rot" in m) and any("scaling" in m["rot"] for t, m in mixers if "rot" in m)
    assert {0.0, 1.0} <= {d for t, m in mixers if t == "lightning" for d in m["decay"]}
    assert any(l["mlp"] is None for l in CONFIG_C["layers"]) and len(CONFIG_D["layers"]) == 6
