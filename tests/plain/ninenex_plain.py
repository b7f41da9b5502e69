"""Ninenex restated from its equations: whole sequences, no cache, no batching, one function per
mechanism, written with explicit loops where that makes the rule plain.  It shares no code with the
engine; the tests compare the engine with it.

Notation: ``x [T, W]`` is the stream of one sequence, position ``i`` sees position ``j`` of the same
sequence.  ``config`` is the mapping a ``config.json`` holds, ``tensors`` the checkpoint by name.
Everything is computed in the dtype of the tensors handed in (the tests hand in float32 or float64).
"""

from __future__ import annotations

import math

import torch


def centred_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """Layer norm with a weight and nothing added."""
    d = x - x.mean(dim=-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(dim=-1, keepdim=True) + eps) * weight


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """``x / sqrt(mean(x^2) + eps)`` over the last dimension."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def projected(name: str, tensors: dict, h: torch.Tensor) -> torch.Tensor:
    """``W h``, plus the bias where the checkpoint has one."""
    y = h @ tensors[name].T
    return y + tensors[name + ".b"] if name + ".b" in tensors else y


# -- a matrix memory with exponential gates ----------------------------------------------------------


def capped_gates(i_raw: torch.Tensor, f_raw: torch.Tensor, cap: float) -> tuple[torch.Tensor, torch.Tensor]:
    """The logarithms of the input and the forget gate."""
    return cap * torch.tanh(i_raw / cap), torch.nn.functional.logsigmoid(cap * torch.tanh(f_raw / cap))


def least(m: torch.Tensor) -> torch.Tensor:
    """What a read-out is divided by at least."""
    return torch.exp(-m)


def memory_walk(q, k, v, i, f) -> torch.Tensor:
    """One head: ``q, k [T, D]`` (``q`` scaled), ``v [T, Dv]``, log gates ``i, f [T]`` -> ``[T, Dv]``."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=q.dtype)
    n = torch.zeros(q.shape[1], dtype=q.dtype)
    m = torch.zeros((), dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(q.shape[0]):
        top = torch.maximum(f[t] + m, i[t])
        keep, add = torch.exp(f[t] + m - top), torch.exp(i[t] - top)
        m = top
        S = keep * S + add * torch.outer(k[t], v[t])
        n = keep * n + add * k[t]
        out[t] = (S.T @ q[t]) / (torch.maximum((n @ q[t]).abs(), least(m)) + 1e-6)
    return out


def matrix_memory(prefix: str, sizes: dict, tensors: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    T, H, D, Dv = h.shape[0], sizes["heads"], sizes["dim"], sizes["vdim"]
    q = projected(prefix + ".q", tensors, h).view(T, H, D) * D ** -0.5
    k = projected(prefix + ".k", tensors, h).view(T, H, D)
    v = projected(prefix + ".v", tensors, h).view(T, H, Dv)
    i, f = capped_gates(projected(prefix + ".i", tensors, h), projected(prefix + ".f", tensors, h), sizes["gate_cap"])
    o = torch.stack([memory_walk(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a]) for a in range(H)], dim=1)
    o = unit_rms(o, eps).reshape(T, H * Dv) * tensors[prefix + ".norm"]
    return (o * torch.sigmoid(projected(prefix + ".g", tensors, h))) @ tensors[prefix + ".o"].T


# -- attention in chunks -----------------------------------------------------------------------------


def turn_halves(x: torch.Tensor, rot: dict) -> torch.Tensor:
    """``x [T, heads, D]``: elements ``i`` and ``i + dims/2`` of the first ``dims`` form a pair; at position ``p``
    the pair ``(u, v)`` becomes ``(u cos a - v sin a, v cos a + u sin a)``, ``a = p base^(-2i/dims)``."""
    out, half = x.clone(), rot["dims"] // 2
    for i in range(half):
        angle = torch.arange(x.shape[0], dtype=torch.float64) * rot["base"] ** (-2.0 * i / rot["dims"])
        c, s = angle.cos().to(x.dtype)[:, None], angle.sin().to(x.dtype)[:, None]
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def sees(i: int, j: int, chunk: int | None) -> bool:
    return j <= i and (chunk is None or i // chunk == j // chunk)


def chunked_heads(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, chunk: int | None) -> torch.Tensor:
    """``q [T, H, D]``, ``k [T, G, D]``, ``v [T, G, Dv]`` -> ``[T, H * Dv]``."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    visible = torch.tensor([[sees(i, j, chunk) for j in range(T)] for i in range(T)])
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for head in range(H):
        g = head // (H // G)
        scores = (q[:, head] @ k[:, g].T * scale).masked_fill(~visible, -math.inf)
        out[:, head] = torch.softmax(scores, dim=1) @ v[:, g]
    return out.reshape(T, -1)


def chunked_attention(prefix: str, sizes: dict, tensors: dict, h: torch.Tensor) -> torch.Tensor:
    T, H, G = h.shape[0], sizes["heads"], sizes["kv_heads"]
    q = projected(prefix + ".q", tensors, h).view(T, H, sizes["dim"])
    k = projected(prefix + ".k", tensors, h).view(T, G, sizes["dim"])
    v = projected(prefix + ".v", tensors, h).view(T, G, sizes["vdim"])
    if sizes.get("rot"):
        q, k = turn_halves(q, sizes["rot"]), turn_halves(k, sizes["rot"])
    chunk = sizes["mask"]["size"] if sizes.get("mask") else None
    return projected(prefix + ".o", tensors, chunked_heads(q, k, v, sizes["scale"], chunk))


# -- retention ---------------------------------------------------------------------------------------


def retention_walk(q, k, v, decay: float) -> torch.Tensor:
    """One head: ``S <- decay S + k v^T``, ``o = S^T q``."""
    S = torch.zeros(q.shape[1], v.shape[1], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(q.shape[0]):
        S = decay * S + torch.outer(k[t], v[t])
        out[t] = S.T @ q[t]
    return out


def retention(prefix: str, sizes: dict, tensors: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    T, H, D, Dv = h.shape[0], sizes["heads"], sizes["dim"], sizes["vdim"]
    q = (h @ tensors[prefix + ".q"].T).view(T, H, D)
    k = (h @ tensors[prefix + ".k"].T).view(T, H, D) * D ** -0.5
    v = (h @ tensors[prefix + ".v"].T).view(T, H, Dv)
    o = torch.stack([retention_walk(q[:, a], k[:, a], v[:, a], sizes["decay"][a]) for a in range(H)], dim=1)
    o = unit_rms(o, eps).reshape(T, H * Dv)
    return (o * silu(h @ tensors[prefix + ".g"].T)) @ tensors[prefix + ".o"].T


def side_by_side(prefix: str, sizes: dict, tensors: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    return (sizes["left_scale"] * chunked_attention(prefix + ".left", sizes["left"], tensors, h)
            + sizes["right_scale"] * retention(prefix + ".right", sizes["right"], tensors, h, eps))


# -- feed-forwards -----------------------------------------------------------------------------------


def gated_unit(prefix: str, tensors: dict, h: torch.Tensor, act) -> torch.Tensor:
    return projected(prefix + ".down", tensors, act(projected(prefix + ".gate", tensors, h)) * projected(prefix + ".up", tensors, h))


def chosen(z: torch.Tensor, top: int) -> list[tuple[int, float]]:
    """The experts of one token with their weights: the softmax over the largest ``top`` logits alone."""
    order = sorted(range(len(z)), key=lambda e: (-float(z[e]), e))[:top]
    return list(zip(order, torch.softmax(z[order], dim=0)))


def experts(prefix: str, sizes: dict, tensors: dict, h: torch.Tensor) -> torch.Tensor:
    z = projected(prefix + ".router", tensors, h)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, weight in chosen(z[t], sizes["router"]["top"]):
            out[t] += weight * gated_unit(f"{prefix}.e{e}", tensors, h[t], silu)
    return out + gated_unit(prefix + ".shared", tensors, h, silu) if sizes.get("shared") else out


def feed_forward(prefix: str, sizes: dict, tensors: dict, h: torch.Tensor) -> torch.Tensor:
    return gated_unit(prefix, tensors, h, gelu_tanh) if sizes["kind"] == "dense" else experts(prefix, sizes, tensors, h)


# -- the model ---------------------------------------------------------------------------------------


def tensors_of(config: dict, index: int) -> int:
    """The layer whose tensors layer ``index`` uses."""
    while config["layers"][index].get("weights_of") is not None:
        index = config["layers"][index]["weights_of"]
    return index


def streams(config: dict, tensors: dict, tokens: list[int]) -> list[torch.Tensor]:
    """The stream behind the embedding and behind every layer."""
    eps = config["norm"]["eps"]
    x = tensors["embed"][torch.tensor(tokens)] * config["embedding"]["scale"]
    out = [x]
    for index, layer in enumerate(config["layers"]):
        p = f"l{tensors_of(config, index)}"
        h = centred_norm(x, tensors[p + ".norm1"], eps)
        mixer = matrix_memory if layer["type"] == "mlstm" else side_by_side
        x = x + centred_norm(mixer(p + ".mix", layer["mixer"], tensors, h, eps), tensors[p + ".norm1b"], eps)
        if layer.get("mlp"):
            h = centred_norm(x, tensors[p + ".norm2"], eps)
            x = x + centred_norm(feed_forward(p + ".mlp", layer["mlp"], tensors, h), tensors[p + ".norm2b"], eps)
        out.append(x)
    return out


def forward(config: dict, tensors: dict, tokens: list[int]) -> torch.Tensor:
    """``[T, V]`` logits of every position."""
    x = streams(config, tensors, tokens)[-1]
    return centred_norm(x, tensors["final.norm"], config["norm"]["eps"]) @ tensors["head"].T * config["logit_scale"]
