"""Plain whole-sequence implementation of the Losivik design, for tests.

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


def softplus(x: torch.Tensor) -> torch.Tensor:
    return torch.log1p(torch.exp(-x.abs())) + x.clamp(min=0)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(
        math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def relu2(z: torch.Tensor) -> torch.Tensor:
    return z.clamp(min=0) ** 2


def linear(W: Weights, name: str, x: torch.Tensor) -> torch.Tensor:
    return x @ W[name].double().t()


def norm_around_zero(W: Weights, name: str, x: torch.Tensor, eps: float
                     ) -> torch.Tensor:
    """The stored weight is the difference from 1."""
    return unit(x, eps) * (1.0 + W[name].double())


# ------------------------------------------------------------- embedding

def position_vectors(T: int, width: int) -> torch.Tensor:
    """[T, width]: entries 2i and 2i + 1 are sin and cos of
    p 10000^(-2i / width)."""
    out = torch.zeros(T, width, dtype=F64)
    for p in range(T):
        for c in range(width):
            a = p * 10000.0 ** (-2.0 * (c // 2) / width)
            out[p, c] = math.cos(a) if c % 2 else math.sin(a)
    return out


def embedding(cfg: dict, W: Weights, tokens: List[int]) -> torch.Tensor:
    x = W["embed"].double()[torch.tensor(list(tokens))]
    return x * float(cfg["embedding"]["scale"]) + \
        position_vectors(len(tokens), int(cfg["width"]))


# ------------------------------------------------------------- attention

def visible(T: int, mask: dict) -> torch.Tensor:
    """[T, T], row sees key: the last `size` tokens, itself included, and
    the first keep_first tokens of the sequence."""
    i = torch.arange(T)
    d = i[:, None] - i[None, :]
    near = (d >= 0) & (d < int(mask["size"]))
    return near | ((d >= 0) & (i[None, :] < int(mask.get("keep_first", 0))))


def softmax_rows(s: torch.Tensor, ok: torch.Tensor) -> torch.Tensor:
    s = s.masked_fill(~ok, float("-inf"))
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def latent_attention(W: Weights, p: str, m: dict, h: torch.Tensor,
                     eps: float) -> torch.Tensor:
    """Keys and values of every head are projections of one normed latent
    per token; no positions; a gate per head on the output."""
    T = h.shape[0]
    H, D, V = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = linear(W, p + "q", h).view(T, H, D)
    c = unit(linear(W, p + "dkv", h), eps) * W[p + "dkv.norm"].double()
    k = linear(W, p + "uk", c).view(T, H, D)
    v = linear(W, p + "uv", c).view(T, H, V)
    g = sigmoid(linear(W, p + "g", h))
    ok = visible(T, {"size": m["mask"]["size"]})
    out = torch.zeros(T, H, V, dtype=F64)
    for n in range(H):
        s = q[:, n] @ k[:, n].t() * float(m["scale"])
        out[:, n] = softmax_rows(s, ok) @ v[:, n] * g[:, n : n + 1]
    return linear(W, p + "o", out.reshape(T, H * V))


def grouped_attention(W: Weights, p: str, m: dict, h: torch.Tensor,
                      eps: float) -> torch.Tensor:
    """Grouped-query attention with normed queries and keys and a window
    that also keeps the first tokens."""
    T = h.shape[0]
    H, G, D, V = (int(m[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    q = unit(linear(W, p + "q", h).view(T, H, D), eps) * \
        W[p + "q.norm"].double()
    k = unit(linear(W, p + "k", h).view(T, G, D), eps) * \
        W[p + "k.norm"].double()
    v = linear(W, p + "v", h).view(T, G, V)
    ok = visible(T, m["mask"])
    out = torch.zeros(T, H, V, dtype=F64)
    for n in range(H):
        g = n // (H // G)
        s = q[:, n] @ k[:, g].t() * float(m["scale"])
        out[:, n] = softmax_rows(s, ok) @ v[:, g]
    return linear(W, p + "o", out.reshape(T, H * V))


# ----------------------------------------------- state-space recurrence

def causal_conv(u: torch.Tensor, w: torch.Tensor, b: torch.Tensor
                ) -> torch.Tensor:
    """u [T, C], w [C, taps], b [C]: y_t = b + sum_j w[:, j]
    u_(t - taps + 1 + j), zeros before the start."""
    T, taps = u.shape[0], w.shape[1]
    y = b[None, :].expand(T, -1).clone()
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j] * u[s]
    return y


def ssd_scan(x, B, C, dt, rate, D):
    """x [T, H, V], B, C [T, H, N] (each head's own group), dt [T, H], rate,
    D [H] -> y [T, H, V]. Per token and head: fade the N x V memory by
    exp(-rate dt), add dt B x^T, read with C, add D x."""
    T, H, V = x.shape
    S = torch.zeros(H, B.shape[-1], V, dtype=F64)
    y = torch.zeros(T, H, V, dtype=F64)
    for t in range(T):
        for n in range(H):
            S[n] = math.exp(-float(rate[n]) * float(dt[t, n])) * S[n] + \
                float(dt[t, n]) * torch.outer(B[t, n], x[t, n])
            y[t, n] = S[n].t() @ C[t, n] + D[n] * x[t, n]
    return y


def state_space(W: Weights, p: str, m: dict, h: torch.Tensor, eps: float
                ) -> torch.Tensor:
    T = h.shape[0]
    H, V, N, G = (int(m[k]) for k in ("heads", "vdim", "state", "groups"))
    inner = H * V
    z, xbc, dt = linear(W, p + "in", h).split(
        [inner, inner + 2 * G * N, H], dim=-1)
    xbc = silu(causal_conv(xbc, W[p + "conv"].double(),
                           W[p + "conv.b"].double()))
    x, B, C = xbc.split([inner, G * N, G * N], dim=-1)
    own = [n // (H // G) for n in range(H)]
    y = ssd_scan(x.view(T, H, V), B.view(T, G, N)[:, own],
                 C.view(T, G, N)[:, own],
                 softplus(dt + W[p + "dt_bias"].double()),
                 torch.exp(W[p + "A_log"].double()), W[p + "D"].double())
    y = y.reshape(T, inner) * silu(z)
    k = int(m["norm_groups"])
    y = unit(y.view(T, k, inner // k), eps).view(T, inner) * \
        W[p + "norm"].double()
    return linear(W, p + "o", y)


def parallel(W: Weights, p: str, m: dict, h: torch.Tensor, eps: float
             ) -> torch.Tensor:
    left = grouped_attention(W, p + "left.", m["left"], h, eps)
    right = state_space(W, p + "right.", m["right"], h, eps)
    return float(m["left_scale"]) * left + float(m["right_scale"]) * right


MIXERS = {"latent_attention": latent_attention, "parallel": parallel}


# ---------------------------------------------------------- feed-forward

def dense(W: Weights, p: str, f: dict, h: torch.Tensor) -> torch.Tensor:
    """Clamped gated unit with biases."""
    lim = float(f["limit"])
    g = (linear(W, p + "gate", h) + W[p + "gate.b"].double()).clamp(max=lim)
    u = (linear(W, p + "up", h) + W[p + "up.b"].double()).clamp(-lim, lim)
    return linear(W, p + "down", g * sigmoid(1.702 * g) * (u + 1.0)) + \
        W[p + "down.b"].double()


def route(W: Weights, p: str, r: dict, h: torch.Tensor
          ) -> Tuple[torch.Tensor, torch.Tensor]:
    """(chosen experts [T, top], their weights)."""
    s = sigmoid(linear(W, p + "router", h))
    w, idx = s.topk(int(r["top"]), dim=-1)
    return idx, w


def expert(W: Weights, p: str, h: torch.Tensor) -> torch.Tensor:
    return linear(W, p + "down", relu2(linear(W, p + "up", h)))


def moe(W: Weights, p: str, f: dict, h: torch.Tensor) -> torch.Tensor:
    """The routing weight scales what an expert reads."""
    idx, w = route(W, p, f["router"], h)
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for j in range(idx.shape[1]):
            y[t] += expert(W, f"{p}e{int(idx[t, j])}.", w[t, j] * h[t])
    if f.get("shared"):
        y = y + expert(W, p + "shared.", h)
    return y


# ----------------------------------------------------- token side input

def token_side(cfg: dict, W: Weights, i: int, x: torch.Tensor,
               tokens: List[int], eps: float) -> torch.Tensor:
    """What layer i adds to the residual from its part of the per-token
    side table."""
    dim, p = int(cfg["token_side"]["dim"]), f"l{i}.side."
    e = W["side.embed"].double()[torch.tensor(list(tokens))]
    e = e[:, i * dim : (i + 1) * dim]
    y = linear(W, p + "proj", gelu_tanh(linear(W, p + "gate", x)) * e)
    return unit(y, eps) * W[p + "norm"].double()


# ----------------------------------------------------------------- model

def forward(cfg: dict, W: Weights, tokens: List[int],
            layers: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab]; `layers` (a list) receives the residual after
    every layer."""
    eps = float(cfg["norm"]["eps"])
    x = embedding(cfg, W, tokens)
    for i, l in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = W[p + "ls1"].double() * MIXERS[l["type"]](
            W, p + "mix.", l["mixer"],
            norm_around_zero(W, p + "norm1", x, eps), eps)
        f = l.get("mlp")
        if f:
            ff = dense if f["kind"] == "dense" else moe
            y = y + W[p + "ls2"].double() * ff(
                W, p + "mlp.", f, norm_around_zero(W, p + "norm2", x, eps))
        x = x + y
        x = x + token_side(cfg, W, i, x, tokens, eps)
        if layers is not None:
            layers.append(x.clone())
    return linear(W, "embed", norm_around_zero(W, "final.norm", x, eps))


# ----------------------------------------------------- small checkpoints

def make_config(*, kinds=("parallel", "latent_attention", "parallel",
                          "latent_attention"),
                mlps=("moe", "dense", None, "moe"), vocab=70, width=22,
                eps=1e-5, embed_scale=3.0, side=7, lat_heads=3, lat_dim=5,
                lat_vdim=4, kv_rank=11, lat_window=6, lat_scale=0.4,
                heads=4, kv_heads=2, dim=6, vdim=5, window=9, keep=3,
                scale=0.37, left_scale=0.8, right_scale=1.3, ssd_heads=4,
                ssd_vdim=6, state=7, groups=2, norm_groups=3, conv=4,
                ff=12, limit=1.5, experts=5, top=2, expert_ff=10,
                shared_ff=8) -> dict:
    mixers = {
        "latent_attention": {"heads": lat_heads, "dim": lat_dim,
                             "vdim": lat_vdim, "kv_rank": kv_rank,
                             "scale": lat_scale,
                             "mask": {"size": lat_window}},
        "parallel": {
            "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                     "vdim": vdim, "scale": scale,
                     "mask": {"size": window, "keep_first": keep}},
            "right": {"heads": ssd_heads, "vdim": ssd_vdim, "state": state,
                      "groups": groups, "norm_groups": norm_groups,
                      "conv": conv},
            "left_scale": left_scale, "right_scale": right_scale}}
    moe_cfg = {"kind": "moe", "expert": {"ff": expert_ff},
               "router": {"experts": experts, "top": top}}
    if shared_ff:
        moe_cfg["shared"] = {"ff": shared_ff}
    table = {"dense": {"kind": "dense", "ff": ff, "limit": limit},
             "moe": moe_cfg, None: None}
    return {"architecture": "Losivik", "vocab": vocab, "width": width,
            "embedding": {"scale": embed_scale}, "norm": {"eps": eps},
            "token_side": {"dim": side},
            "layers": [{"type": k, "mixer": json.loads(json.dumps(mixers[k])),
                        "mlp": table[f] and dict(table[f])}
                       for k, f in zip(kinds, mlps)]}


def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    """Checkpoint names and shapes of a config."""
    Wd, n, e = int(cfg["width"]), len(cfg["layers"]), cfg["token_side"]["dim"]
    out: Dict[str, tuple] = {"embed": (cfg["vocab"], Wd),
                             "side.embed": (cfg["vocab"], n * e),
                             "final.norm": (Wd,)}
    for i, l in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.mix.", l["mixer"], l.get("mlp")
        for k in ("1", "2") if f else ("1",):
            out[f"l{i}.norm{k}"] = out[f"l{i}.ls{k}"] = (Wd,)
        out.update({f"l{i}.side.gate": (e, Wd), f"l{i}.side.proj": (Wd, e),
                    f"l{i}.side.norm": (Wd,)})
        if l["type"] == "latent_attention":
            H, D, V, C = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
            out.update({p + "q": (H * D, Wd), p + "dkv": (C, Wd),
                        p + "dkv.norm": (C,), p + "uk": (H * D, C),
                        p + "uv": (H * V, C), p + "g": (H, Wd),
                        p + "o": (Wd, H * V)})
        else:
            a, q = m["left"], p + "left."
            H, G, D, V = (a[k] for k in ("heads", "kv_heads", "dim", "vdim"))
            out.update({q + "q": (H * D, Wd), q + "k": (G * D, Wd),
                        q + "v": (G * V, Wd), q + "q.norm": (D,),
                        q + "k.norm": (D,), q + "o": (Wd, H * V)})
            a, q = m["right"], p + "right."
            H, V, N, G = (a[k] for k in ("heads", "vdim", "state", "groups"))
            ch = H * V + 2 * G * N
            out.update({q + "in": (H * V + ch + H, Wd),
                        q + "conv": (ch, a["conv"]), q + "conv.b": (ch,),
                        q + "dt_bias": (H,), q + "A_log": (H,), q + "D": (H,),
                        q + "norm": (H * V,), q + "o": (Wd, H * V)})
        if not f:
            continue
        p = f"l{i}.mlp."
        if f["kind"] == "dense":
            for name, s in (("gate", (f["ff"], Wd)), ("up", (f["ff"], Wd)),
                            ("down", (Wd, f["ff"]))):
                out[p + name], out[p + name + ".b"] = s, s[:1]
            continue
        out[p + "router"] = (f["router"]["experts"], Wd)
        parts = [(f"e{k}.", f["expert"]["ff"])
                 for k in range(f["router"]["experts"])]
        if f.get("shared"):
            parts.append(("shared.", f["shared"]["ff"]))
        for name, ff in parts:
            out[p + name + "up"], out[p + name + "down"] = (ff, Wd), (Wd, ff)
    return out


def random_weights(cfg: dict, seed: int) -> Weights:
    gen = torch.Generator().manual_seed(seed)
    W = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(shape, generator=gen)
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1", "norm2") or name == "final.norm":
            t = 0.3 * t                     # around zero
        elif last == "norm":
            t = 1.0 + 0.3 * t
        elif last in ("ls1", "ls2"):
            t = 0.7 + 0.3 * t
        elif last == "b":
            t = 0.3 * t
        elif last == "A_log":
            t = -0.5 + t
        elif last == "dt_bias":
            t = -1.0 + t
        elif last == "conv":
            t = 0.5 * t
        elif last == "D":
            t = 1.0 + 0.5 * t
        elif name == "embed":
            t = 0.4 * t
        elif name != "side.embed":
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
