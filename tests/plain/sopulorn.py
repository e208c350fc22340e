"""The Sopulorn decoder written out plainly in float64, one function a mechanism.

Nothing here is shared with the product: the tests compare the engine's logits with these.
A model is ``(config mapping, name -> float64 tensor)``; the config mapping is config.json's.
Whole sequences, no cache: every function sees all ``T`` tokens of one request.
"""

from __future__ import annotations

import math

import torch

F = torch.float64


def over_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def offset_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """RMS norm whose stored weight is the gain's distance from one."""
    return over_rms(x, eps) * (1.0 + w)


def bigram_rows(tokens, bigram: dict) -> list[int]:
    """The row of the bigram table that every token adds; the first token takes the row behind the buckets."""
    rows = []
    for i, token in enumerate(tokens):
        if i == 0:
            rows.append(bigram["buckets"])
        else:
            rows.append((int(tokens[i - 1]) * bigram["mul_prev"] + int(token) * bigram["mul_cur"]) % bigram["buckets"])
    return rows


def embedding(config: dict, weights: dict, tokens) -> torch.Tensor:
    x = weights["embed"][torch.as_tensor(list(tokens), dtype=torch.long)]
    bigram = (config.get("embedding") or {}).get("bigram")
    if bigram:
        x = x + weights["bigram"][torch.tensor(bigram_rows(tokens, bigram), dtype=torch.long)]
    return x


def rotate(x: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """``x [T, heads, d]``, row t at position t: pairs ``(i, i + dims / 2)`` of the first ``dims`` turned."""
    half = dims // 2
    out = x.clone()
    for i in range(half):
        angle = torch.arange(x.shape[0], dtype=F) * base ** (-2.0 * i / dims)
        c, s = torch.cos(angle)[:, None], torch.sin(angle)[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


def softmax_with_one(scores: torch.Tensor) -> torch.Tensor:
    """Causal weights of ``scores [T, T]``; the denominator holds one more term, the exponential of zero."""
    T = scores.shape[0]
    scores = scores.masked_fill(torch.arange(T)[None, :] > torch.arange(T)[:, None], -math.inf)
    top = torch.clamp(scores.max(-1, keepdim=True).values, min=0.0)
    e = torch.exp(scores - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(-top))


def heads_of(h: torch.Tensor, w: dict, name: str, heads: int, dim: int) -> torch.Tensor:
    return (h @ w[name].T + w[name + ".b"]).view(h.shape[0], heads, dim)


def rotation_of(m: dict) -> tuple[int, float]:
    rot = m.get("rot")
    return (rot["dims"], rot["base"]) if rot else (0, 1.0)


def keys_and_values(h: torch.Tensor, w: dict, m: dict, eps: float) -> tuple[torch.Tensor, torch.Tensor]:
    """What a layer with projections of its own puts into the cache."""
    k = over_rms(heads_of(h, w, "k", m["kv_heads"], m["dim"]), eps) * w["k.norm"]
    return rotate(k, *rotation_of(m)), heads_of(h, w, "v", m["kv_heads"], m["vdim"])


def attention(h: torch.Tensor, w: dict, m: dict, eps: float, kv: tuple[torch.Tensor, torch.Tensor]) -> torch.Tensor:
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = over_rms(heads_of(h, w, "q", H, m["dim"]), eps) * w["q.norm"]
    q = rotate(q, *rotation_of(m))
    k, v = kv
    out = torch.zeros(T, H, v.shape[-1], dtype=F)
    for head in range(H):
        g = head // (H // G)
        out[:, head] = softmax_with_one((q[:, head] @ k[:, g].T) * m["scale"]) @ v[:, g]
    return out.reshape(T, -1) @ w["o"].T


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def dense_ff(h: torch.Tensor, w: dict, mlp: dict) -> torch.Tensor:
    limit = mlp["limit"]
    g = torch.clamp(h @ w["gate"].T, max=limit)
    u = torch.clamp(h @ w["up"].T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w["down"].T


def expert(h: torch.Tensor, w: dict, name: str) -> torch.Tensor:
    return (silu(h @ w[name + ".gate"].T) * (h @ w[name + ".up"].T)) @ w[name + ".down"].T


def route(h: torch.Tensor, w: dict, router: dict) -> tuple[torch.Tensor, torch.Tensor]:
    """``(choice [T, top], weight [T, top])``: the largest logits, weights by a softmax over them alone."""
    z = h @ w["router"].T + w["router.b"]
    best = z.topk(router["top"], dim=-1)
    return best.indices, torch.softmax(best.values, dim=-1)


def routed_ff(h: torch.Tensor, w: dict, mlp: dict) -> torch.Tensor:
    choice, weight = route(h, w, mlp["router"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for c in range(choice.shape[1]):
            out[t] += weight[t, c] * expert(h[t: t + 1], w, f"e{int(choice[t, c])}")[0]
    if mlp.get("shared"):
        out = out + torch.sigmoid(h @ w["shared.sg"].T) * expert(h, w, "shared")
    return out


def sub(weights: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(config: dict, weights: dict, tokens, stream_after=None) -> torch.Tensor:
    """Logits ``[T, vocab]`` for one request.  ``stream_after``: a list that receives the stream
    after every layer."""
    eps = config["norm"]["eps"]
    x = embedding(config, weights, tokens)
    held: dict[int, tuple[torch.Tensor, torch.Tensor]] = {}
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        w = sub(weights, p + "mix.")
        h = offset_norm(x, weights[p + "norm1"], eps)
        if m.get("kv_from") is None:
            held[i] = keys_and_values(h, w, m, eps)
        else:
            held[i] = held[m["kv_from"]]
        x = x + offset_norm(attention(h, w, m, eps, held[i]), weights[p + "norm1b"], eps)
        mlp = layer.get("mlp")
        if mlp:
            w = sub(weights, p + "mlp.")
            h = offset_norm(x, weights[p + "norm2"], eps)
            y = dense_ff(h, w, mlp) if mlp["kind"] == "dense" else routed_ff(h, w, mlp)
            x = x + offset_norm(y, weights[p + "norm2b"], eps)
        if stream_after is not None:
            stream_after.append(x.clone())
    return offset_norm(x, weights["final.norm"], eps) @ weights["head"].T
