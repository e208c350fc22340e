"""Configurations and model folders for the Sopulorn tests.

The configurations differ from each other in every size and option: head counts and grouping, key
and value sizes (equal, half, double, neither), how much of a head is rotated, which layers keep keys
and values and which read another's, clamps, experts with and without a shared one, layers without a
feed-forward, the pair table, and values that are 1 or equal where another model's differ.
"""

from __future__ import annotations

from pathlib import Path

import torch


def attn(heads, kv, dim, vdim, scale, rot=None, base=10000.0, kv_from=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}
    if rot != 0:
        m["rot"] = {"dims": dim if rot is None else rot, "base": base}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(ff, experts, top, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def layer(mixer, mlp):
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def model(vocab, width, eps, bigram, layers):
    out = {"architecture": "Sopulorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if bigram:
        out["embedding"] = {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}
    return out


# two layers with keys and values of their own, of different sizes, each read by a later one with
# another scale; part of a head rotated; pages of 8
CONFIG_A = model(211, 96, 1e-5, (101, 7, 29), [
    layer(attn(4, 2, 24, 40, 0.2, 16, 500.0), dense(80, 0.6)),
    layer(attn(3, 3, 16, 16, 0.25), moe(24, 12, 3, 40)),
    layer(attn(4, 2, 24, 40, 0.3, 16, 500.0, kv_from=0), moe(40, 5, 2)),
    layer(attn(3, 3, 16, 16, 0.15, kv_from=1), None),
    layer(attn(6, 2, 16, 24, 0.3, 8), dense(136, 1.5)),
])

# the shapes that the matrix-core attention kernels serve in bfloat16 (pages of 16): keys of 64 with
# values of 32, 64 and 128, keys of 128 with values of 64, all or part of a head rotated, each read
# by another layer
CONFIG_B = model(320, 128, 1e-6, (513, 3000, 4097), [
    layer(attn(4, 2, 64, 32, 0.14), dense(192, 1.0)),
    layer(attn(4, 4, 128, 64, 0.1, 64), moe(64, 8, 2, 96)),
    layer(attn(4, 4, 128, 64, 0.07, 64, kv_from=1), moe(32, 16, 4, 64)),
    layer(attn(6, 2, 64, 64, 0.12, 32), moe(64, 4, 1, 32)),
    layer(attn(4, 2, 64, 32, 0.2, kv_from=0), dense(64, 0.4)),
    layer(attn(2, 1, 64, 128, 0.13), None),
    layer(attn(6, 2, 64, 64, 0.1, 32, kv_from=3), moe(32, 8, 3)),
])

# ones and equal values: one head, values of one element, two rotated elements and none, one bucket
# (every pair the same row), one expert, all experts chosen, an odd vocabulary
CONFIG_C = model(97, 40, 1e-4, (1, 5, 0), [
    layer(attn(1, 1, 8, 1, 1.0, 2), moe(8, 1, 1, 8)),
    layer(attn(2, 1, 8, 8, 0.5, 0), moe(8, 3, 3)),
    layer(attn(1, 1, 8, 1, 1.0, 2, kv_from=0), dense(8, 1.0)),
    layer(attn(2, 2, 6, 10, 0.5), None),
])

# no pair table; sixteen query heads on one key head, keys of 32 with values of 16, of 96 with 48, of
# 256 with 128, of 280; a chain of readers of one layer
CONFIG_D = model(256, 64, 1e-6, None, [
    layer(attn(16, 1, 32, 16, 0.2), dense(24, 0.3)),
    layer(attn(4, 2, 96, 48, 0.12, 50), moe(16, 6, 2, 48)),
    layer(attn(16, 1, 32, 16, 0.25, kv_from=0), moe(32, 9, 4, 16)),
    layer(attn(32, 1, 32, 16, 0.15, kv_from=0), dense(40, 2.0)),
    layer(attn(2, 1, 256, 128, 0.06, 128), None),
    layer(attn(3, 1, 280, 72, 0.06, 30), moe(16, 2, 2, 8)),
])

CONFIGS = {"A": (CONFIG_A, 8), "B": (CONFIG_B, 16), "C": (CONFIG_C, 4), "D": (CONFIG_D, 16)}


def random_config(rng) -> dict:
    """A configuration drawn from ``rng`` (a ``random.Random``): two to seven layers, every size and
    constant drawn anew."""
    width = rng.choice([64, 96, 128, 192, 256, 100, 72])
    layers, owners = [], []
    for i in range(rng.randint(2, 7)):
        scale = rng.choice([0.125, 0.2, 0.09])
        if owners and rng.random() < 0.4:
            j = rng.choice(owners)
            m = dict(layers[j]["mixer"], scale=scale, kv_from=j)
        else:
            kv, dim = rng.choice([1, 2, 3, 4]), rng.choice([64, 64, 128, 32, 96, 48, 24, 40])
            vdim = rng.choice([dim // 2, dim // 2, dim, 2 * dim, 24, 80])
            rot = rng.choice([dim, dim, dim // 2 // 2 * 2, 2, 0])
            m = attn(kv * rng.choice([1, 2, 4]), kv, dim, vdim, scale, rot, rng.choice([500.0, 10000.0, 1e6]))
            owners.append(i)
        r = rng.random()
        if r < 0.12:
            f = None
        elif r < 0.45:
            f = dense(rng.choice([24, 32, 64, 96, 40, 136]), rng.choice([0.3, 1.0, 2.5, 7.0]))
        else:
            experts = rng.choice([1, 2, 5, 8, 16, 33])
            f = moe(rng.choice([16, 24, 32, 64, 40]), experts, rng.randint(1, min(experts, 5)),
                    rng.choice([None, 16, 32, 64, 40]))
        layers.append(layer(m, f))
    bigram = None if rng.random() < 0.15 else (rng.choice([1, 37, 128, 1000]), rng.choice([1, 43, 100003, 0]),
                                               rng.choice([1, 19, 65537]))
    return model(rng.choice([97, 256, 512, 1000]), width, rng.choice([1e-6, 1e-5]), bigram, layers)


def make_model_dir(folder: Path, config: dict, seed: int) -> Path:
    """A model folder from the product's random-weights mode, with the tensors redrawn so that each
    one matters: norms' stored weights lie around zero (heads' gains around one), biases are felt, the
    pairs' rows are as large as the tokens', the dense feed-forward reaches its clamps, and the
    matrices are livelier than N(0, 0.02)."""
    from safetensors.torch import load_file, save_file

    from kvcore_amd.weights.loader import write_random_model

    write_random_model(folder, config, seed)
    path = folder / "model.safetensors"
    tensors = load_file(str(path))
    gen = torch.Generator().manual_seed(seed + 1)

    def noise(t, std, mean=0.0):
        return (torch.randn(t.shape, generator=gen) * std + mean).to(torch.bfloat16).to(t.dtype)

    for name, t in list(tensors.items()):
        parts = name.split(".")
        leaf = parts[-1]
        if name.endswith(("q.norm", "k.norm")):
            tensors[name] = noise(t, 0.2, 1.0)
        elif leaf.startswith("norm"):
            tensors[name] = noise(t, 0.2)
        elif leaf == "b":
            tensors[name] = noise(t, 0.4)
        elif name in ("embed", "bigram"):
            tensors[name] = noise(t, 0.6)
        elif leaf in ("router", "sg"):
            tensors[name] = noise(t, 2.0 * t.shape[1] ** -0.5)
        elif t.dim() == 2:
            tensors[name] = noise(t, 1.2 * t.shape[1] ** -0.5)
    save_file(tensors, str(path))
    return folder
