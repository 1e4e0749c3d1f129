"""Plain, slow implementation of the Vugudra design, one function per mechanism, token by token where
recurrent. It shares no code with ``vgate`` and is what tests/test_vugudra.py holds the engine against.

Everything is float64 (``dt``) on the CPU; ``cfg`` is the parsed config.json, ``t`` a dict name -> tensor.
"""
from __future__ import annotations

import math

import torch

dt = torch.float64


def rms(x: torch.Tensor, eps: float, w: torch.Tensor | None = None) -> torch.Tensor:
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w.to(dt)


def lin(w: torch.Tensor, x: torch.Tensor) -> torch.Tensor:
    return x @ w.to(dt).t()


def silu(x: torch.Tensor) -> torch.Tensor:
    return x / (1.0 + torch.exp(-x))


def softplus(x: torch.Tensor) -> torch.Tensor:
    return torch.clamp(x, min=0.0) + torch.log1p(torch.exp(-x.abs()))


def frequencies(dims: int, base: float, scaling: dict | None = None) -> tuple:
    """([dims / 2] angular frequencies, the factor on cos and sin). ``scaling``: frequencies whose wavelength fits
    ``fast`` or more times into ``original`` positions stay, those that fit ``slow`` or fewer times are divided by
    ``factor``, linear in the index between."""
    f = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return f, 1.0
    s = float(scaling["factor"])

    def index(turns):
        return dims * math.log(scaling["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    a = max(math.floor(index(scaling["fast"])), 0)
    b = min(math.ceil(index(scaling["slow"])), dims - 1)
    out = []
    for i, x in enumerate(f):
        r = min(max((i - a) / max(b - a, 0.001), 0.0), 1.0)
        out.append(x / s * r + x * (1.0 - r))
    return out, 0.1 * math.log(s) + 1.0


def turn(x: torch.Tensor, pos: torch.Tensor, dims: int, rot: dict, half: bool) -> torch.Tensor:
    """x [n, ..., d]: the first ``dims`` entries in pairs (i, i + dims / 2) or (2i, 2i + 1), turned by their angles."""
    f, amp = frequencies(dims, rot["base"], rot.get("scaling"))
    y = x.clone()
    for i in range(dims // 2):
        a = pos.to(dt) * f[i]
        shape = [x.shape[0]] + [1] * (x.dim() - 2)
        c, s = (torch.cos(a) * amp).view(shape), (torch.sin(a) * amp).view(shape)
        i0, i1 = (i, i + dims // 2) if half else (2 * i, 2 * i + 1)
        u, v = x[..., i0], x[..., i1]
        y[..., i0] = u * c - v * s
        y[..., i1] = v * c + u * s
    return y


def sink_softmax(s: torch.Tensor, sink: float | None) -> torch.Tensor:
    """Weights over the last axis of ``s``; with a sink the denominator has exp(sink) once more."""
    m = s.max(-1, keepdim=True).values
    if sink is not None:
        m = torch.clamp(m, min=float(sink))
    e = torch.exp(s - m)
    den = e.sum(-1, keepdim=True)
    if sink is not None:
        den = den + torch.exp(torch.tensor(float(sink), dtype=dt) - m)
    return e / den


def seen(n: int, size: int, first: int) -> torch.Tensor:
    """[n, n] bool: position i sees j <= i that is nearer than ``size`` or one of the ``first`` first."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    return (j <= i) & ((i - j < size) | (j < first))


def latent_attention(m: dict, t: dict, eps: float, h: torch.Tensor) -> torch.Tensor:
    n = h.shape[0]
    H, D, R, V, K = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(n)
    q = lin(t["uq"], rms(lin(t["dq"], h), eps, t["dq.norm"])).view(n, H, D + R)
    kv = lin(t["dkv"], h)
    c = rms(kv[:, :K], eps, t["dkv.norm"])
    qr = turn(q[..., D:], pos, m["rot"]["dims"], m["rot"], True)
    kr = turn(kv[:, K:], pos, m["rot"]["dims"], m["rot"], True)
    k, v = lin(t["uk"], c).view(n, H, D), lin(t["uv"], c).view(n, H, V)
    gate = torch.sigmoid(lin(t["g"], h))
    causal = seen(n, n + 1, 0)
    out = torch.zeros(n, H, V, dtype=dt)
    for hd in range(H):
        s = (q[:, hd, :D] @ k[:, hd].t() + qr[:, hd] @ kr.t()) * m["scale"]
        p = sink_softmax(s.masked_fill(~causal, float("-inf")), float(t["sink"][hd]))
        out[:, hd] = (p @ v[:, hd]) * gate[:, hd: hd + 1]
    return lin(t["o"], out.reshape(n, H * V))


def window_attention(m: dict, t: dict, eps: float, h: torch.Tensor) -> torch.Tensor:
    """The cached value of a token is its key as projected."""
    n = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    pos = torch.arange(n)
    kp = lin(t["k"], h).view(n, G, D)
    q = turn(rms(lin(t["q"], h).view(n, H, D), eps, t["q.norm"]), pos, m["rot"]["dims"], m["rot"], False)
    k = turn(rms(kp, eps, t["k.norm"]), pos, m["rot"]["dims"], m["rot"], False)
    vis = seen(n, m["mask"]["size"], m["mask"]["keep_first"])
    out = torch.zeros(n, H, D, dtype=dt)
    for hd in range(H):
        g = hd // (H // G)
        s = (q[:, hd] @ k[:, g].t()) * m["scale"]
        out[:, hd] = sink_softmax(s.masked_fill(~vis, float("-inf")), None) @ kp[:, g]
    return lin(t["o"], out.reshape(n, H * D))


def short_conv(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor | None) -> torch.Tensor:
    """x [n, C], w [C, taps]: y_t = b + sum_i w[:, i] x_(t - taps + 1 + i), zeros before the start; then silu."""
    n, taps = x.shape[0], w.shape[1]
    w = w.to(dt)
    y = torch.zeros_like(x) if b is None else b.to(dt).expand_as(x).clone()
    for i in range(taps):
        back = taps - 1 - i
        if back < n:
            y[back:] += w[:, i] * x[: n - back]
    return silu(y)


def gated_delta(m: dict, t: dict, eps: float, h: torch.Tensor) -> torch.Tensor:
    n = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    unit = lambda x: x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)  # noqa: E731
    q = unit(short_conv(lin(t["q"], h), t["q.conv"], None).view(n, G, D)) * D ** -0.5
    k = unit(short_conv(lin(t["k"], h), t["k.conv"], None).view(n, G, D))
    v = short_conv(lin(t["v"], h), t["v.conv"], None).view(n, H, V)
    beta = torch.sigmoid(lin(t["b"], h))
    g = lin(t["a2"], lin(t["a1"], h)) + t["dt_bias"].to(dt)
    g = torch.exp(-torch.exp(t["A_log"].to(dt))[None, :, None] * softplus(g).view(n, H, D))
    S = torch.zeros(H, D, V, dtype=dt)
    out = torch.zeros(n, H, V, dtype=dt)
    for i in range(n):
        for hd in range(H):
            ki, qi = k[i, hd // (H // G)], q[i, hd // (H // G)]
            s = g[i, hd][:, None] * S[hd]
            u = beta[i, hd] * (v[i, hd] - s.t() @ ki)
            S[hd] = s + ki[:, None] * u[None, :]
            out[i, hd] = S[hd].t() @ qi
    out = rms(out, eps, t["norm"]) * torch.sigmoid(lin(t["g2"], lin(t["g1"], h))).view(n, H, V)
    return lin(t["o"], out.reshape(n, H * V))


def parallel(m: dict, t: dict, eps: float, h: torch.Tensor) -> torch.Tensor:
    a = window_attention(m["left"], sub(t, "left."), eps, h)
    b = gated_delta(m["right"], sub(t, "right."), eps, h)
    return 0.5 * (rms(a, eps, t["left.out"]) + rms(b, eps, t["right.out"]))


def mamba1(m: dict, t: dict, eps: float, h: torch.Tensor) -> torch.Tensor:
    n = h.shape[0]
    C, N, R = m["inner"], m["state"], m["dt_rank"]
    xz = lin(t["in"], h)
    x, z = short_conv(xz[:, :C], t["conv"], t["conv.b"]), xz[:, C:]
    p = lin(t["x"], x)
    d = softplus(lin(t["dt"], p[:, :R]) + t["dt.b"].to(dt))
    B, Cc = p[:, R: R + N], p[:, R + N:]
    A = -torch.exp(t["A_log"].to(dt))
    S = torch.zeros(C, N, dtype=dt)
    y = torch.zeros(n, C, dtype=dt)
    for i in range(n):
        S = torch.exp(d[i][:, None] * A) * S + (d[i] * x[i])[:, None] * B[i][None, :]
        y[i] = S @ Cc[i] + t["D"].to(dt) * x[i]
    return lin(t["o"], y * silu(z))


def feed_forward(m: dict, t: dict, h: torch.Tensor) -> torch.Tensor:
    return lin(t["down"], silu(lin(t["gate"], h)) * lin(t["up"], h))


MIXERS = {"latent_attention": latent_attention, "parallel": parallel, "mamba1": mamba1}


def sub(t: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in t.items() if k.startswith(prefix)}


def run_order(cfg: dict) -> list:
    n = len(cfg["layers"])
    lp = cfg.get("loop") or {"start": 0, "stop": 0, "times": 0}
    mid = list(range(lp["start"], lp["stop"]))
    return list(range(lp["start"])) + mid * lp["times"] + list(range(lp["stop"], n))


def forward(cfg: dict, t: dict, tokens: list) -> tuple:
    """(logits [n, vocab], residual stream after every layer run [runs, n, W])."""
    eps = cfg["norm"]["eps"]
    x = t["embed"].to(dt)[torch.tensor(tokens)]
    streams = []
    for i in run_order(cfg):
        L = cfg["layers"][i]
        lt = sub(t, f"l{i}.")
        y = MIXERS[L["type"]](L["mixer"], sub(lt, "mix."), eps, rms(x, eps, 1.0 + lt["norm1"].to(dt)))
        if L.get("mlp"):
            y = y + feed_forward(L["mlp"], sub(lt, "mlp."), rms(x, eps, 1.0 + lt["norm2"].to(dt)))
        x = x + y
        streams.append(x.clone())
    return lin(t["head"], rms(x, eps, 1.0 + t["final.norm"].to(dt))), torch.stack(streams)
