"""The Zikupel decoder written out plainly in float64, one function a mechanism.

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


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def relu_squared(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0.0) ** 2


# ------------------------------------------------------------------------ positions
def turns_dim(t: float, dims: int, base: float, original: float) -> float:
    """The (fractional) pair that turns ``t`` times over ``original`` positions."""
    return dims * math.log(original / (2 * math.pi * t)) / (2 * math.log(base))


def frequencies(rot: dict) -> tuple[list[float], float]:
    """A frequency per pair, and the factor on cosine and sine."""
    dims, base = rot["dims"], rot["base"]
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if not s:
        return plain, 1.0
    lo = max(math.floor(turns_dim(s["fast"], dims, base, s["original"])), 0)
    hi = min(math.ceil(turns_dim(s["slow"], dims, base, s["original"])), dims - 1)
    out = []
    for i, f in enumerate(plain):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * ramp + f * (1.0 - ramp))
    return out, 0.1 * math.log(s["factor"]) + 1.0


def rotate(x: torch.Tensor, rot: dict | None) -> torch.Tensor:
    """``x [T, heads, d]``, row t at position t: pairs ``(i, i + dims / 2)`` of the first ``dims`` turned."""
    if not rot or not rot["dims"]:
        return x
    freqs, factor = frequencies(rot)
    half = rot["dims"] // 2
    out = x.clone()
    for i, f in enumerate(freqs):
        angle = torch.arange(x.shape[0], dtype=F) * f
        c, s = (torch.cos(angle) * factor)[:, None], (torch.sin(angle) * factor)[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


# ------------------------------------------------------------------------ attention
def capped(scores: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(scores / cap)


def causal_softmax(scores: torch.Tensor) -> torch.Tensor:
    T = scores.shape[0]
    return torch.softmax(scores.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), -math.inf), -1)


def projected_heads(h: torch.Tensor, w: dict, name: str, heads: int, dim: int) -> torch.Tensor:
    return (h @ w[name].T + w[name + ".b"]).view(h.shape[0], heads, dim)


def attention(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    raw = projected_heads(h, w, "k", G, m["dim"])
    q = rotate(over_rms(projected_heads(h, w, "q", H, m["dim"]), eps) * w["q.norm"], m.get("rot"))
    k = rotate(over_rms(raw, eps) * w["k.norm"], m.get("rot"))
    v = raw  # the values are the keys as projected
    out = torch.zeros(T, H, m["dim"], dtype=F)
    for head in range(H):
        g = head // (H // G)
        s = (q[:, head] @ k[:, g].T) * m["scale"]
        if m.get("softcap"):
            s = capped(s, m["softcap"])
        out[:, head] = causal_softmax(s) @ v[:, g]
    return (out.reshape(T, -1) * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


# ------------------------------------------------------------------------ lightning
def lightning_state(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay) -> torch.Tensor:
    """``q, k [T, heads, d]``, ``v [T, heads, dv]``, a number per head: ``S <- decay S + k v^T; o = S^T q``."""
    T, H, d = q.shape
    out = torch.zeros(T, H, v.shape[-1], dtype=F)
    for head in range(H):
        S = torch.zeros(d, v.shape[-1], dtype=F)
        for t in range(T):
            S = decay[head] * S + torch.outer(k[t, head], v[t, head])
            out[t, head] = S.T @ q[t, head]
    return out


def lightning(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    T, H = h.shape[0], m["heads"]
    q = silu(h @ w["q"].T).view(T, H, m["dim"])
    k = silu(h @ w["k"].T).view(T, H, m["dim"])
    v = silu(h @ w["v"].T).view(T, H, m["vdim"])
    o = lightning_state(q, k, v, m["decay"]).reshape(T, -1)
    return (over_rms(o, eps) * w["norm"] * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


# --------------------------------------------------------------------- feed-forward
def dense_ff(h: torch.Tensor, w: dict) -> torch.Tensor:
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def expert(h: torch.Tensor, w: dict, name: str) -> torch.Tensor:
    return relu_squared(h @ w[name + ".up"].T) @ w[name + ".down"].T


def route(h: torch.Tensor, w: dict, top: int) -> tuple[torch.Tensor, torch.Tensor]:
    """``(choice [T, top], weight [T, top])``: the largest sigmoids, as they are."""
    best = torch.sigmoid(h @ w["router"].T).topk(top, dim=-1)
    return best.indices, best.values


def routed_ff(h: torch.Tensor, w: dict, mlp: dict) -> torch.Tensor:
    choice, weight = route(h, w, mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for c in range(choice.shape[1]):  # the weight is on the expert's input
            out[t] += expert(weight[t, c] * h[t: t + 1], w, f"e{int(choice[t, c])}")[0]
    if mlp.get("shared"):
        out = out + expert(h, w, "shared")
    return out


# ---------------------------------------------------------------------------- model
def sub(weights: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(config: dict, weights: dict, tokens, stream_after=None) -> torch.Tensor:
    """Logits ``[T, vocab]`` for one request.  ``stream_after``: a list that receives the stream
    after every layer."""
    eps = config["norm"]["eps"]
    x = weights["embed"][torch.as_tensor(list(tokens), dtype=torch.long)]
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}."
        mixer = {"attention": attention, "lightning": lightning}[layer["type"]]
        x = x + offset_norm(mixer(x, sub(weights, p + "mix."), layer["mixer"], eps), weights[p + "norm1"], eps)
        mlp = layer.get("mlp")
        if mlp:
            w = sub(weights, p + "mlp.")
            y = dense_ff(x, w) if mlp["kind"] == "dense" else routed_ff(x, w, mlp)
            x = x + offset_norm(y, weights[p + "norm2"], eps)
        if stream_after is not None:
            stream_after.append(x.clone())
    return offset_norm(x, weights["final.norm"], eps) @ weights["head"].T
