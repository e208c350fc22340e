"""Configurations and model folders for the Zikupel tests.

The configurations differ from each other in every size and option: head counts and grouping, key
sizes that the matrix-core kernels serve and others, how much of a head is rotated and with which
frequencies, soft caps on either side of what needs a running maximum and none, key and value sizes of
the lightning layers, slow and fast decays, experts with and without a shared one, layers without a
feed-forward, and values that are 1 or equal where another model's differ.
"""

from __future__ import annotations

from pathlib import Path

import torch


def yarn(factor, original, fast, slow):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def attn(heads, kv, dim, scale, softcap=None, rot=None, base=10000.0, scaling=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale}
    if softcap is not None:
        m["softcap"] = softcap
    if rot != 0:
        m["rot"] = {"dims": dim if rot is None else rot, "base": base}
        if scaling is not None:
            m["rot"]["scaling"] = scaling
    return "attention", m


def lightning(dim, vdim, *decay):
    return "lightning", {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def layer(mixer, mlp):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}


def model(vocab, width, eps, layers):
    return {"architecture": "Zikupel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


# sizes that only the general kernels serve; pages of 8
CONFIG_A = model(211, 96, 1e-5, [
    layer(attn(4, 2, 24, 0.5, 5.0, 16, 500.0, yarn(4.0, 64, 8.0, 1.0)), dense(80)),
    layer(lightning(24, 40, 0.97, 0.5, 0.999), moe(24, 12, 3, 40)),
    layer(attn(3, 3, 16, 0.4, None, 0), moe(40, 5, 2)),
    layer(lightning(10, 5, 0.9, 0.995), None),
    layer(attn(6, 1, 40, 1.2, 50.0, 8), dense(136)),
])

# the shapes that the matrix-core attention kernels serve in bfloat16 (pages of 16)
CONFIG_B = model(320, 128, 1e-6, [
    layer(attn(4, 2, 64, 0.3, 8.0, 64, 10000.0, yarn(8.0, 256, 32.0, 1.0)), dense(192)),
    layer(lightning(64, 64, 0.9, 0.99, 0.999, 0.6), moe(64, 8, 2, 96)),
    layer(attn(4, 1, 128, 0.2, 60.0, 32, 1000.0), moe(32, 16, 4, 64)),
    layer(attn(8, 8, 64, 0.25, 20.0, 48, 500.0, yarn(2.0, 32, 4.0, 0.5)), moe(64, 4, 1, 32)),
    layer(lightning(128, 32, 0.98, 0.2), dense(64)),
    layer(attn(6, 2, 64, 0.4, 3.0, 0), None),
    layer(attn(4, 2, 64, 0.2, None, 16), moe(32, 8, 3)),
])

# ones and equal values: one head, keys and values of one element, a decay of one and of zero, a cap of
# one, two rotated elements and none, one expert, all experts chosen, an odd vocabulary
CONFIG_C = model(97, 40, 1e-4, [
    layer(lightning(1, 1, 1.0), moe(8, 1, 1, 8)),
    layer(attn(1, 1, 8, 1.0, 1.0, 2), moe(8, 3, 3)),
    layer(lightning(8, 8, 0.0, 1.0, 0.5), dense(8)),
    layer(attn(2, 1, 6, 0.5, 2.0, 0), None),
    layer(lightning(4, 12, 0.9), None),
])

# sixteen query heads on one key head, keys of 32, 96, 256 and 280, lightning keys of 200 and 256
CONFIG_D = model(256, 64, 1e-6, [
    layer(attn(16, 1, 32, 0.4, 10.0), dense(24)),
    layer(lightning(200, 72, 0.95, 0.99), moe(16, 6, 2, 48)),
    layer(attn(4, 2, 96, 0.2, 44.0, 50, 10000.0, yarn(16.0, 128, 16.0, 2.0)), moe(32, 9, 4, 16)),
    layer(attn(2, 1, 256, 0.12, 15.0, 128), None),
    layer(lightning(256, 16, 0.999, 0.8, 0.97, 0.4), dense(40)),
    layer(attn(3, 1, 280, 0.1, 12.0, 30), moe(16, 2, 2, 8)),
])

CONFIGS = {"A": (CONFIG_A, 8), "B": (CONFIG_B, 16), "C": (CONFIG_C, 4), "D": (CONFIG_D, 16)}


def random_config(rng) -> dict:
    """A configuration drawn from ``rng`` (a ``random.Random``): two to seven layers, every size and
    constant drawn anew."""
    layers = []
    for _ in range(rng.randint(2, 7)):
        if rng.random() < 0.4:
            m = lightning(rng.choice([4, 16, 24, 30, 32, 64, 100, 128]), rng.choice([1, 8, 20, 32, 64, 96, 130]),
                          *(rng.choice([0.3, 0.8, 0.97, 0.99, 0.999]) for _ in range(rng.choice([1, 2, 3, 5]))))
        else:
            kv, dim = rng.choice([1, 2, 3, 4]), rng.choice([64, 64, 128, 32, 96, 48, 24, 40])
            rot = rng.choice([dim, dim // 2 // 2 * 2, 16, 2, 0])
            scaling = rng.choice([None, yarn(rng.choice([2.0, 8.0, 40.0]), rng.choice([32, 100, 1000]),
                                             rng.choice([4.0, 32.0]), rng.choice([0.5, 1.0, 2.0]))])
            m = attn(kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([0.125, 0.3, 0.6]),
                     rng.choice([None, 2.0, 10.0, 30.0, 70.0]), rot, rng.choice([500.0, 10000.0, 1e6]), scaling)
        r = rng.random()
        if r < 0.12:
            f = None
        elif r < 0.35:
            f = dense(rng.choice([24, 32, 64, 96, 40, 136]))
        else:
            experts = rng.choice([1, 2, 5, 8, 12, 33])
            f = moe(rng.choice([16, 24, 32, 64, 40]), experts, rng.randint(1, min(experts, 5)),
                    rng.choice([None, 16, 32, 64, 40]))
        layers.append(layer(m, f))
    return model(rng.choice([97, 256, 512, 1000]), rng.choice([64, 96, 128, 256, 100, 72]), rng.choice([1e-6, 1e-5]), layers)


def make_model_dir(folder: Path, config: dict, seed: int) -> Path:
    """A model folder from the product's random-weights mode, with the tensors redrawn so that each
    one matters: norms' stored weights lie around zero (the heads' and the lightning norm's gains around
    one), biases are felt, and the matrices are livelier than N(0, 0.02)."""
    from safetensors.torch import load_file, save_file

    from kvcore_amd.weights.loader import write_random_model

    write_random_model(folder, config, seed)
    path = folder / "model.safetensors"
    tensors = load_file(str(path))
    gen = torch.Generator().manual_seed(seed + 1)

    def noise(t, std, mean=0.0):
        return (torch.randn(t.shape, generator=gen) * std + mean).to(torch.bfloat16).to(t.dtype)

    for name, t in list(tensors.items()):
        leaf = name.split(".")[-1]
        if leaf == "norm" and ".mix." in name:
            tensors[name] = noise(t, 0.2, 1.0)
        elif leaf.startswith("norm"):
            tensors[name] = noise(t, 0.2)
        elif leaf == "b":
            tensors[name] = noise(t, 0.4)
        elif name == "embed":
            tensors[name] = noise(t, 0.8)
        elif leaf == "router":
            tensors[name] = noise(t, 1.5 * t.shape[1] ** -0.5)
        elif t.dim() == 2:
            tensors[name] = noise(t, 1.2 * t.shape[1] ** -0.5)
    save_file(tensors, str(path))
    return folder
