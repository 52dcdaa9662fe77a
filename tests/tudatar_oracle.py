"""Plain whole-sequence implementation of the Tudatar design, for tests.

One function per mechanism, float64, no cache, no batching, no chunking, and
no code shared with the serving path (bee2bee_amd.*). Inputs: the parsed
config.json dict and a dict of checkpoint-named tensors.

Notation: unit(x) = x / sqrt(mean(x^2) + eps) over the last axis; row t of a
[T, ...] tensor is position t of one sequence.
"""
from __future__ import annotations

import json
import math
import os
from typing import Dict, List, Optional, Tuple

import torch

F64 = torch.float64
Weights = Dict[str, torch.Tensor]


def unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(x: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x: torch.Tensor) -> torch.Tensor:
    return x * sigmoid(x)


def linear(W: Weights, name: str, x: torch.Tensor) -> torch.Tensor:
    return x @ W[name].double().t()


# ------------------------------------------------------------------ norm

def tanh_norm(W: Weights, name: str, x: torch.Tensor) -> torch.Tensor:
    """tanh(alpha x) * w + b: no statistics over the row."""
    a = W[name + ".alpha"].double()
    return torch.tanh(a * x) * W[name].double() + W[name + ".b"].double()


# -------------------------------------------------------------- rotation

def rotation(rot: dict) -> Tuple[List[float], float]:
    """(angular frequency of every rotated pair, factor on cos and sin).
    With a 'scaling' entry the slow pairs turn `factor` times slower, the
    fast ones as they are, with a linear ramp over the pair index between
    the two indices at which a pair completes `fast` / `slow` turns within
    `original` positions."""
    n, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    factor, orig = float(sc["factor"]), float(sc["original"])

    def index(turns: float) -> float:
        return n * math.log(orig / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(index(float(sc["fast"]))), 0)
    hi = min(math.ceil(index(float(sc["slow"]))), n - 1)
    out = []
    for i, x in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(x / factor * r + x * (1.0 - r))
    return out, 0.1 * math.log(factor) + 1.0


def rotate_pairs(x: torch.Tensor, freq: List[float], mag: float
                 ) -> torch.Tensor:
    """x [T, heads, R]: coordinate 2i turns with 2i+1; coordinates past the
    rotated ones pass."""
    out = x.clone()
    pos = torch.arange(x.shape[0], dtype=F64)
    for i, f in enumerate(freq):
        c = (torch.cos(pos * f) * mag)[:, None]
        s = (torch.sin(pos * f) * mag)[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i] = u * c - v * s
        out[:, :, 2 * i + 1] = v * c + u * s
    return out


# ---------------------------------------------------------------- mixers

def visible(T: int, window: Optional[int]) -> torch.Tensor:
    i = torch.arange(T)
    d = i[:, None] - i[None, :]
    ok = d >= 0
    if window:
        ok = ok & (d < window)
    return ok


def softmax_rows(s: torch.Tensor, ok: torch.Tensor) -> torch.Tensor:
    s = s.masked_fill(~ok, float("-inf"))
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def latent_attention(W: Weights, p: str, m: dict, h: torch.Tensor,
                     eps: float) -> torch.Tensor:
    """Keys and values are up-projections of a shared normed latent; a
    rotated part of each query meets one rotated key part shared by all
    heads."""
    T = h.shape[0]
    H, D, R, V, C = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim",
                                         "kv_rank"))
    cq = unit(linear(W, p + "dq", h), eps) * W[p + "dq.norm"].double()
    q = linear(W, p + "uq", cq).view(T, H, D + R)
    ckv = linear(W, p + "dkv", h)
    c = unit(ckv[:, :C], eps) * W[p + "dkv.norm"].double()
    freq, mag = rotation(m["rot"])
    kr = rotate_pairs(ckv[:, None, C:], freq, mag)[:, 0]
    qr = rotate_pairs(q[:, :, D:], freq, mag)
    kn = linear(W, p + "uk", c).view(T, H, D)
    vv = linear(W, p + "uv", c).view(T, H, V)
    ok = visible(T, None)
    out = torch.zeros(T, H, V, dtype=F64)
    for n in range(H):
        s = (q[:, n, :D] @ kn[:, n].t() + qr[:, n] @ kr.t()) * float(m["scale"])
        out[:, n] = softmax_rows(s, ok) @ vv[:, n]
    return linear(W, p + "o", out.reshape(T, H * V))


def distance_bias(r1: float, r2: float, T: int) -> torch.Tensor:
    """What is taken off the score of (row i, key j <= i):
    r1 ln(1 + r2 (i - j))."""
    i = torch.arange(T, dtype=F64)
    d = (i[:, None] - i[None, :]).clamp(min=0)
    return r1 * torch.log(1.0 + r2 * d)


def attention(W: Weights, p: str, m: dict, h: torch.Tensor, eps: float
              ) -> torch.Tensor:
    """Windowed grouped-query attention without rotation: q and k normed
    over the whole projection, values normed per head, scores lowered with
    the logarithm of the distance."""
    T = h.shape[0]
    H, G, D, V = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))

    def proj(n):
        return linear(W, p + n, h) + W[p + n + ".b"].double()

    q = (unit(proj("q"), eps) * W[p + "q.norm"].double()).view(T, H, D)
    k = (unit(proj("k"), eps) * W[p + "k.norm"].double()).view(T, G, D)
    v = unit(proj("v").view(T, G, V), eps)
    ok = visible(T, int((m.get("mask") or {}).get("size", 0) or 0))
    out = torch.zeros(T, H, V, dtype=F64)
    for n in range(H):
        g = n // (H // G)
        s = q[:, n] @ k[:, g].t() * float(m["scale"])
        s = s - distance_bias(float(W[p + "r1"][n]), float(W[p + "r2"][n]), T)
        out[:, n] = softmax_rows(s, ok) @ v[:, g]
    return linear(W, p + "o", out.reshape(T, H * V))


def short_conv(u: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros
    before the start."""
    T, taps = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j] * u[s]
    return y


def unit_length(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def channel_decay(W: Weights, p: str, h: torch.Tensor, H: int, D: int
                  ) -> torch.Tensor:
    """[T, H, D] fade of each head's memory rows."""
    a = linear(W, p + "a2", linear(W, p + "a1", h)) + W[p + "dt_bias"].double()
    sp = torch.log1p(torch.exp(-a.abs())) + a.clamp(min=0)     # softplus
    rate = torch.exp(W[p + "A_log"].double())
    return torch.exp(-rate[None, :, None] * sp.view(-1, H, D))


def delta_scan(q, k, v, beta, g):
    """q, k [T, H, D], v [T, H, V], beta [T, H], g [T, H, D] -> [T, H, V].
    Per token: fade the rows, take what the key recalls out of the write,
    write, read."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=F64)
    out = []
    for t in range(T):
        S = g[t][:, :, None] * S
        for n in range(H):
            u = beta[t, n] * (v[t, n] - S[n].t() @ k[t, n])
            S[n] = S[n] + torch.outer(k[t, n], u)
        out.append(torch.stack([S[n].t() @ q[t, n] for n in range(H)]))
    return torch.stack(out)


def channel_delta(W: Weights, p: str, m: dict, h: torch.Tensor, eps: float
                  ) -> torch.Tensor:
    T = h.shape[0]
    H, G, D, V = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))

    def part(n):
        return silu(short_conv(linear(W, p + n, h), W[p + n + ".conv"].double()))

    q = unit_length(part("q").view(T, G, D)) * D ** -0.5
    k = unit_length(part("k").view(T, G, D))
    v = part("v").view(T, H, V)
    own = [n // (H // G) for n in range(H)]
    o = delta_scan(q[:, own], k[:, own], v, sigmoid(linear(W, p + "b", h)),
                   channel_decay(W, p, h, H, D))
    gate = sigmoid(linear(W, p + "g2", linear(W, p + "g1", h))).view(T, H, V)
    y = unit(o, eps) * W[p + "norm"].double() * gate
    return linear(W, p + "o", y.reshape(T, H * V))


MIXERS = {"latent_attention": latent_attention, "attention": attention,
          "channel_delta": channel_delta}


# ---------------------------------------------------------- feed-forward

def route(W: Weights, p: str, r: dict, h: torch.Tensor
          ) -> Tuple[torch.Tensor, torch.Tensor]:
    """(chosen experts [T, top], their weights)."""
    s = sigmoid(linear(W, p + "router", h))
    pick = s + W[p + "correction"].double()
    idx = pick.topk(int(r["top"]), dim=-1).indices
    w = s.gather(1, idx)
    return idx, w / (w.sum(-1, keepdim=True) + 1e-20) * float(r["scale"])


def expert(W: Weights, p: str, h: torch.Tensor) -> torch.Tensor:
    return linear(W, p + "down", silu(linear(W, p + "gate", h)) *
                  linear(W, p + "up", h))


def moe(W: Weights, p: str, f: dict, h: torch.Tensor) -> torch.Tensor:
    idx, w = route(W, p, f["router"], h)
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(idx.shape[1]):
            y[t] += w[t, j] * expert(W, f"{p}e{int(idx[t, j])}.", h[t])
    return y


# ----------------------------------------------------------------- model

def forward(cfg: dict, W: Weights, tokens: List[int],
            layers: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab]; `layers` (a list) receives the residual after
    every layer."""
    eps = float(cfg["norm"]["eps"])
    x = W["embed"].double()[torch.tensor(list(tokens))]
    for i, l in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = MIXERS[l["type"]](W, p + "mix.", l["mixer"],
                              tanh_norm(W, p + "norm1", x), eps)
        x = x + tanh_norm(W, p + "norm1b", y)
        if l.get("mlp"):
            y = moe(W, p + "mlp.", l["mlp"], tanh_norm(W, p + "norm2", x))
            x = x + tanh_norm(W, p + "norm2b", y)
        if layers is not None:
            layers.append(x.clone())
    return linear(W, "head", tanh_norm(W, "final.norm", x)) * \
        float(cfg["logit_scale"])


# ----------------------------------------------------- small checkpoints

def make_config(*, kinds=("channel_delta", "attention", "latent_attention",
                          "attention"), vocab=70, width=22, eps=1e-5,
                logit_scale=0.6, heads=4, kv_heads=2, dim=6, vdim=5,
                window=9, scale=0.37, lat_heads=3, lat_dim=5, rot_dim=6,
                lat_vdim=4, kv_rank=11, q_rank=9, lat_scale=0.4, base=300.0,
                scaling=True, delta_heads=4, delta_kv=2, delta_dim=7,
                delta_vdim=6, conv=3, experts=5, top=2, ff=10, rscale=1.7,
                no_mlp=()) -> dict:
    sc = {"factor": 3.0, "original": 40, "fast": 4.0, "slow": 1.0}
    if isinstance(scaling, dict):
        sc = scaling
    rot = {"base": base, "dims": rot_dim}
    if scaling:
        rot["scaling"] = sc
    mixers = {
        "attention": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "scale": scale, "mask": {"size": window}},
        "latent_attention": {"heads": lat_heads, "dim": lat_dim,
                             "rot_dim": rot_dim, "vdim": lat_vdim,
                             "kv_rank": kv_rank, "q_rank": q_rank,
                             "scale": lat_scale, "rot": rot},
        "channel_delta": {"heads": delta_heads, "kv_heads": delta_kv,
                          "dim": delta_dim, "vdim": delta_vdim,
                          "conv": conv}}
    mlp = {"kind": "moe", "expert": {"ff": ff},
           "router": {"experts": experts, "top": top, "scale": rscale}}
    return {"architecture": "Tudatar", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "logit_scale": logit_scale,
            "layers": [{"type": k, "mixer": dict(mixers[k]),
                        "mlp": None if i in no_mlp else dict(mlp)}
                       for i, k in enumerate(kinds)]}


def tensor_shapes(cfg: dict, a_rank: int = 5, g_rank: int = 7
                  ) -> Dict[str, tuple]:
    """Checkpoint names and shapes of a config; a_rank / g_rank are the
    widths of the low-rank decay and gate projections."""
    Wd = int(cfg["width"])
    out: Dict[str, tuple] = {"embed": (cfg["vocab"], Wd),
                             "head": (cfg["vocab"], Wd)}

    def norm(n):
        out[n], out[n + ".b"], out[n + ".alpha"] = (Wd,), (Wd,), ()

    norm("final.norm")
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", l["mixer"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b")
                                        if l.get("mlp") else ()):
            norm(f"l{i}.{n}")
        H, V = m["heads"], m["vdim"]
        out[p + "o"] = (Wd, H * V)
        if l["type"] == "latent_attention":
            D, R, C, Q = m["dim"], m["rot_dim"], m["kv_rank"], m["q_rank"]
            out.update({p + "dq": (Q, Wd), p + "dq.norm": (Q,),
                        p + "uq": (H * (D + R), Q), p + "dkv": (C + R, Wd),
                        p + "dkv.norm": (C,), p + "uk": (H * D, C),
                        p + "uv": (H * V, C)})
        else:
            G, D = m["kv_heads"], m["dim"]
            if l["type"] == "attention":
                sizes = {"q": H * D, "k": G * D, "v": G * V}
                for n, s in sizes.items():
                    out[p + n], out[p + n + ".b"] = (s, Wd), (s,)
                out.update({p + "q.norm": (H * D,), p + "k.norm": (G * D,),
                            p + "r1": (H,), p + "r2": (H,)})
            else:
                sizes = {"q": G * D, "k": G * D, "v": H * V}
                for n, s in sizes.items():
                    out[p + n], out[p + n + ".conv"] = (s, Wd), (s, m["conv"])
                out.update({p + "b": (H, Wd), p + "A_log": (H,),
                            p + "norm": (V,), p + "a1": (a_rank, Wd),
                            p + "a2": (H * D, a_rank),
                            p + "dt_bias": (H * D,), p + "g1": (g_rank, Wd),
                            p + "g2": (H * V, g_rank)})
        f = l.get("mlp")
        if f:
            E, ff = f["router"]["experts"], f["expert"]["ff"]
            p = f"l{i}.mlp."
            out[p + "router"], out[p + "correction"] = (E, Wd), (E,)
            for e in range(E):
                out.update({f"{p}e{e}.gate": (ff, Wd), f"{p}e{e}.up": (ff, Wd),
                            f"{p}e{e}.down": (Wd, ff)})
    return out


def random_weights(cfg: dict, seed: int, a_rank: int = 5, g_rank: int = 7
                   ) -> Weights:
    gen = torch.Generator().manual_seed(seed)
    W = {}
    for name, shape in tensor_shapes(cfg, a_rank, g_rank).items():
        t = torch.randn(shape, generator=gen)
        last = name.rsplit(".", 1)[-1]
        if last == "alpha":
            t = 0.6 + 0.2 * t.clamp(-1.5, 1.5)
        elif last in ("norm", "norm1", "norm1b", "norm2", "norm2b"):
            t = 1.0 + 0.3 * t
        elif last == "b" and len(shape) == 1:
            t = 0.2 * t
        elif last == "correction":
            t = 0.3 * t
        elif last == "r1":
            t = 0.5 + 0.3 * t
        elif last == "r2":
            t = 0.2 + t.abs()
        elif last == "A_log":
            t = -2.0 + t
        elif last == "dt_bias":
            t = -1.0 + t
        elif last == "conv":
            t = 0.5 * t
        elif name not in ("embed",):
            t = t * shape[-1] ** -0.5 * 1.5
        W[name] = t.bfloat16()
    return W


def save_checkpoint(path: str, cfg: dict, W: Weights) -> None:
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    save_file({k: v.contiguous() for k, v in W.items()},
              os.path.join(path, "model.safetensors"))
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
