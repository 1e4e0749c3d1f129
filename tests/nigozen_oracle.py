"""Plain, slow implementation of the Nigozen design, one function per mechanism. It shares no code with
``vgate`` and is what tests/test_nigozen.py holds the engine against.

Everything is float64 (``dt``) on the CPU; ``cfg`` is the parsed config.json, ``t`` a dict name -> tensor.
"""
from __future__ import annotations

import math

import torch

dt = torch.float64


def layer_norm(x: torch.Tensor, eps: float, w: torch.Tensor) -> torch.Tensor:
    """Mean removed, divided by the standard deviation (eps inside the root), weighted; no bias."""
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * w.to(dt)


def lin(w: torch.Tensor, x: torch.Tensor) -> torch.Tensor:
    return x @ w.to(dt).t()


def plus_one_softmax(s: torch.Tensor) -> torch.Tensor:
    """e^s_j / (1 + sum e^s) over the last axis."""
    m = torch.clamp(s.max(-1, keepdim=True).values, min=0.0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def turn_pairs(x: torch.Tensor, pos: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """x [n, heads, d]: entries (2i, 2i + 1) of the first ``dims`` turned by pos * base^(-2i / dims)."""
    y = x.clone()
    for i in range(dims // 2):
        a = (pos.to(dt) * float(base) ** (-2.0 * i / dims)).view(-1, 1)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i] = u * torch.cos(a) - v * torch.sin(a)
        y[..., 2 * i + 1] = v * torch.cos(a) + u * torch.sin(a)
    return y


def visible(n: int, size: int | None) -> torch.Tensor:
    """[n, n] bool: position i (row) sees position j (column)."""
    i, j = torch.arange(n).view(-1, 1), torch.arange(n).view(1, -1)
    ok = j <= i
    return ok if size is None else ok & (i // size == j // size)


def attend(q, k, v, scale: float, size: int | None) -> torch.Tensor:
    """q [n, H, D], k [n, G, D], v [n, G, V] -> [n, H, V]."""
    n, H, G = q.shape[0], q.shape[1], k.shape[1]
    see = visible(n, size)
    out = torch.zeros(n, H, v.shape[2], dtype=dt)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].t()) * scale
        out[:, h] = plus_one_softmax(s.masked_fill(~see, float("-inf"))) @ v[:, g]
    return out


def attention(m: dict, t: dict, h: torch.Tensor, first_values: list) -> torch.Tensor:
    """``first_values``: empty until the first layer that mixes values has put its own there."""
    n = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(n)
    rot = m.get("rot") or {"dims": 0, "base": 1.0}
    q = turn_pairs(lin(t["q"], h).view(n, H, D), pos, rot["dims"], rot["base"])
    k = turn_pairs(lin(t["k"], h).view(n, G, D), pos, rot["dims"], rot["base"])
    v = lin(t["v"], h)
    if m.get("v_mix"):
        if first_values:
            lam = float(t["vmix"].reshape(()))
            v = (1.0 - lam) * v + lam * first_values[0]
        else:
            first_values.append(v)
    size = (m.get("mask") or {}).get("size")
    o = attend(q, k, v.view(n, G, V), m["scale"], size).reshape(n, H * V)
    return lin(t["o"], o * torch.sigmoid(lin(t["g"], h)))


def dense(m: dict, t: dict, h: torch.Tensor) -> torch.Tensor:
    z = lin(t["up"], h)
    return lin(t["down"], z * 0.5 * (1.0 + torch.erf(z / math.sqrt(2.0))))


def experts(m: dict, t: dict, h: torch.Tensor) -> torch.Tensor:
    r = m["router"]
    z = lin(t["router"], h)
    out = torch.zeros_like(h)
    for i in range(h.shape[0]):
        chosen = sorted(range(r["experts"]), key=lambda e: (-float(z[i, e]), e))[: r["top"]]
        w = torch.softmax(z[i, chosen], -1)
        for c, e in enumerate(chosen):
            a = torch.clamp(lin(t[f"e{e}.up"], h[i]), min=0.0)
            out[i] += w[c] * lin(t[f"e{e}.down"], a * a)
    return out


FEED_FORWARDS = {"dense": dense, "moe": experts}


def sub(t: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in t.items() if k.startswith(prefix)}


def forward(cfg: dict, t: dict, tokens: list) -> tuple:
    """(logits [n, vocab], residual stream after every layer [layers, n, W])."""
    eps = cfg["norm"]["eps"]
    x = t["embed"].to(dt)[torch.tensor(tokens)] * cfg["embedding"]["scale"]
    streams, first_values = [], []
    for i, L in enumerate(cfg["layers"]):
        lt = sub(t, f"l{i}.")
        y = attention(L["mixer"], sub(lt, "mix."), layer_norm(x, eps, lt["norm1"]), first_values)
        x = x + layer_norm(y, eps, lt["norm1b"])
        if L.get("mlp"):
            y = FEED_FORWARDS[L["mlp"]["kind"]](L["mlp"], sub(lt, "mlp."), layer_norm(x, eps, lt["norm2"]))
            x = x + layer_norm(y, eps, lt["norm2b"])
        streams.append(x.clone())
    return lin(t["embed"], layer_norm(x, eps, t["final.norm"])), torch.stack(streams)
