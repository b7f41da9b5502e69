"""Lukelix restated from its equations: whole sequences, no cache, no batching, one function per
mechanism, written with explicit loops where that makes the rule plain.  It shares no code with the
engine; the tests compare the engine with it.

Notation: ``x [T, W]`` is the stream of one sequence, position ``i`` sees position ``j`` of the same
sequence.  ``config`` is the mapping a ``config.json`` holds, ``tensors`` the checkpoint by name.
Everything is computed in the dtype of the tensors handed in (the tests hand in float32 or float64).
"""

from __future__ import annotations

import math

import torch


def bigram_rows(tokens: list[int], rule: dict) -> list[int]:
    """Which row of the bigram table each token adds: a hash of the token and the one before it; the row
    behind the hashed ones for a sequence's first token."""
    rows = [rule["buckets"]]
    for before, here in zip(tokens[:-1], tokens[1:]):
        rows.append((before * rule["mul_prev"] + here * rule["mul_cur"]) % rule["buckets"])
    return rows[: len(tokens)]


def embedding(config: dict, tensors: dict, tokens: list[int]) -> torch.Tensor:
    x = tensors["embed"][torch.tensor(tokens)].clone()
    rule = (config.get("embedding") or {}).get("bigram")
    if rule:
        x += tensors["bigram"][torch.tensor(bigram_rows(tokens, rule))]
    return x


def layer_norm(x: torch.Tensor, tensors: dict, name: str, eps: float) -> torch.Tensor:
    mean = x.mean(dim=-1, keepdim=True)
    variance = ((x - mean) ** 2).mean(dim=-1, keepdim=True)
    return (x - mean) / torch.sqrt(variance + eps) * tensors[name] + tensors[name + ".b"]


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """``x / sqrt(mean(x^2) + eps)`` over the last dimension."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def short_conv(u: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """``u [T, C]``, ``taps [C, K]``: ``y_t = sum_j taps[:, j] u_(t - K + 1 + j)``, zeros before the start."""
    T, K = u.shape[0], taps.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(K):
            s = t - K + 1 + j
            if s >= 0:
                y[t] += taps[:, j] * u[s]
    return y


# -- rotation of neighbouring pairs, long wavelengths stretched ------------------------------------


def frequencies(rot: dict) -> list[float]:
    """``f_i`` of the pairs: a frequency whose wave is short against the original length stays, one whose
    wave is long is divided by the factor, those between are blended."""
    out = []
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2.0 * i / rot["dims"])
        stretch = rot.get("scaling")
        if stretch:
            wave = 2 * math.pi / f
            if wave > stretch["original"] / stretch["low"]:
                f = f / stretch["factor"]
            elif wave >= stretch["original"] / stretch["high"]:
                s = (stretch["original"] / wave - stretch["low"]) / (stretch["high"] - stretch["low"])
                f = (1 - s) * f / stretch["factor"] + s * f
        out.append(f)
    return out


def turn_neighbours(x: torch.Tensor, rot: dict) -> torch.Tensor:
    """``x [T, heads, D]``: elements ``2i`` and ``2i + 1`` of the first ``dims`` form a pair; at position ``p``
    the pair ``(u, v)`` becomes ``(u cos a - v sin a, v cos a + u sin a)``, ``a = p f_i``."""
    out = x.clone()
    for i, f in enumerate(frequencies(rot)):
        angle = torch.arange(x.shape[0], dtype=torch.float64) * f
        c, s = angle.cos().to(x.dtype)[:, None], angle.sin().to(x.dtype)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


# -- attention --------------------------------------------------------------------------------------


def projected(which: str, prefix: str, tensors: dict, h: torch.Tensor) -> torch.Tensor:
    """One of q, k, v: projection with bias, then the convolution over time where there is one."""
    u = h @ tensors[f"{prefix}.{which}"].T + tensors[f"{prefix}.{which}.b"]
    taps = tensors.get(f"{prefix}.{which}.conv")
    return u if taps is None else short_conv(u, taps)


def turned_heads(which: str, prefix: str, sizes: dict, heads: int, tensors: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    """Queries or keys ``[T, heads, D]``: projected, normed per head, rotated."""
    x = projected(which, prefix, tensors, h).view(h.shape[0], heads, sizes["dim"])
    x = unit_rms(x, eps) * tensors[f"{prefix}.{which}.norm"]
    return turn_neighbours(x, sizes["rot"]) if sizes.get("rot") else x


def keys_and_values(prefix: str, sizes: dict, tensors: dict, h: torch.Tensor, eps: float) -> tuple[torch.Tensor, torch.Tensor]:
    k = turned_heads("k", prefix, sizes, sizes["kv_heads"], tensors, h, eps)
    v = projected("v", prefix, tensors, h).view(h.shape[0], sizes["kv_heads"], sizes["vdim"])
    return k, v


def softmax_heads(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float) -> torch.Tensor:
    """``q [T, H, D]``, ``k [T, G, D]``, ``v [T, G, Dv]`` -> ``[T, H * Dv]``, position ``i`` over all ``j <= i``."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    hidden = torch.triu(torch.ones(T, T, dtype=torch.bool), 1)
    for head in range(H):
        g = head // (H // G)
        scores = (q[:, head] @ k[:, g].T * scale).masked_fill(hidden, -math.inf)
        out[:, head] = torch.softmax(scores, dim=1) @ v[:, g]
    return out.reshape(T, -1)


def attention(prefix: str, sizes: dict, tensors: dict, h: torch.Tensor, eps: float, kv: dict, index: int) -> torch.Tensor:
    """``kv``: keys and values by the layer that made them."""
    source = sizes.get("kv_from")
    if source is None:
        kv[index] = keys_and_values(prefix, sizes, tensors, h, eps)
        source = index
    q = turned_heads("q", prefix, sizes, sizes["heads"], tensors, h, eps)
    return softmax_heads(q, *kv[source], sizes["scale"]) @ tensors[prefix + ".o"].T


# -- the selective state -----------------------------------------------------------------------------


def selective_walk(x, B, C, dt, rate, skip) -> torch.Tensor:
    """One head: ``x [T, P]``, ``B, C [T, N]``, ``dt [T]``, numbers ``rate``, ``skip``.  The state ``S [N, P]`` starts at
    zero; ``S <- exp(-rate dt) S + dt B x^T``, ``y = S^T C + skip x``."""
    S = torch.zeros(B.shape[1], x.shape[1], dtype=x.dtype)
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(-rate * dt[t]) * S + dt[t] * torch.outer(B[t], x[t])
        y[t] = S.T @ C[t] + skip * x[t]
    return y


def gated_group_norm(y: torch.Tensor, z: torch.Tensor, gain: torch.Tensor, parts: int, eps: float) -> torch.Tensor:
    """``y silu(z)``, every one of ``parts`` equal parts divided by its own root mean square, times ``gain``."""
    gated = y * (z * torch.sigmoid(z))
    T, width = gated.shape
    return unit_rms(gated.view(T, parts, width // parts), eps).reshape(T, width) * gain


def mamba2(prefix: str, sizes: dict, tensors: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    T, H, P, N, G = h.shape[0], sizes["heads"], sizes["vdim"], sizes["state"], sizes["groups"]
    inner = H * P
    z, u, dt = (h @ tensors[prefix + ".in"].T).split([inner, inner + 2 * G * N, H], dim=1)
    u = short_conv(u, tensors[prefix + ".conv"]) + tensors[prefix + ".conv.b"]
    u = u * torch.sigmoid(u)
    x, B, C = u.split([inner, G * N, G * N], dim=1)
    x, B, C = x.view(T, H, P), B.view(T, G, N), C.view(T, G, N)
    dt = torch.nn.functional.softplus(dt + tensors[prefix + ".dt_bias"], threshold=50.0)
    y = torch.zeros(T, H, P, dtype=h.dtype)
    for head in range(H):
        g = head // (H // G)
        rate = math.exp(float(tensors[prefix + ".A_log"][head]))
        y[:, head] = selective_walk(x[:, head], B[:, g], C[:, g], dt[:, head], rate, float(tensors[prefix + ".D"][head]))
    y = gated_group_norm(y.reshape(T, inner), z, tensors[prefix + ".norm"], sizes["norm_groups"], eps)
    return y @ tensors[prefix + ".o"].T


# -- the model ---------------------------------------------------------------------------------------


def feed_forward(prefix: str, tensors: dict, h: torch.Tensor) -> torch.Tensor:
    return torch.relu(h @ tensors[prefix + ".up"].T) ** 2 @ tensors[prefix + ".down"].T


def streams(config: dict, tensors: dict, tokens: list[int]) -> list[torch.Tensor]:
    """The stream behind the embedding and behind every layer."""
    eps = config["norm"]["eps"]
    x = embedding(config, tensors, tokens)
    out = [x]
    kv: dict = {}
    for i, layer in enumerate(config["layers"]):
        prefix, sizes = f"l{i}.mix", layer["mixer"]
        if layer["type"] == "attention":
            mixed = attention(prefix, sizes, tensors, x, eps, kv, i)
        else:
            mixed = mamba2(prefix, sizes, tensors, x, eps)
        x = x + layer_norm(mixed, tensors, f"l{i}.norm1", eps)
        if layer.get("mlp"):
            x = x + layer_norm(feed_forward(f"l{i}.mlp", tensors, x), tensors, f"l{i}.norm2", eps)
        out.append(x)
    return out


def forward(config: dict, tensors: dict, tokens: list[int]) -> torch.Tensor:
    """``[T, V]`` logits of every position."""
    x = streams(config, tensors, tokens)[-1]
    return layer_norm(x, tensors, "final.norm", config["norm"]["eps"]) @ tensors["head"].T
