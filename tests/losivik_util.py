"""Helpers of the Losivik tests: write a small random checkpoint, serve it
with the engine; replay/compare helpers are shared with the other hybrid
families' tests."""
from __future__ import annotations

from typing import Sequence

import torch

from tests import losivik_oracle as O
from tests.nukopel_util import (assert_logits, chunk_schedule,  # noqa: F401
                                random_tokens, rel_err, replay, row_errs)


def make_engine(tmp_path, cfg, W, device="cpu", dtype=torch.float32,
                max_batch=4, block_size=16, kv_blocks=64, max_seq_len=1024,
                **kw):
    from bee2bee_amd.engine.engine import InferenceEngine

    path = str(tmp_path / "ckpt")
    O.save_checkpoint(path, cfg, W)
    return InferenceEngine(
        "lo-test", device=device, dtype=dtype, model_path=path,
        max_batch=max_batch, max_seq_len=max_seq_len,
        use_graphs=kw.pop("use_graphs", False), kv_block_size=block_size,
        kv_blocks=kv_blocks, kv_margin_blocks=1, **kw)


def oracle_logits(cfg, W, tokens: Sequence[int]) -> torch.Tensor:
    return O.forward(cfg, W, list(tokens))


def slow_decay(W, by: float = 6.0):
    """State-space heads that remember for hundreds of tokens."""
    return {k: (v.float() - by).bfloat16() if k.endswith("A_log") else v
            for k, v in W.items()}


def _bare(kind: str, mixer: dict, width: int = 8, vocab: int = 5) -> dict:
    """One layer, no feed-forward, an embedding that outweighs positions."""
    return {"architecture": "Losivik", "vocab": vocab, "width": width,
            "embedding": {"scale": 64.0}, "norm": {"eps": 1e-5},
            "token_side": {"dim": 2},
            "layers": [{"type": kind, "mixer": mixer, "mlp": None}]}


def _planted(cfg, far: int, T: int):
    """(weights, tokens) of a bare config: token ids 0 and 2 everywhere, id 1
    at `far`. The residual starts as [1, is0, is1, is2, 0...] * 64; ids 3
    and 4 read axes 5 and 6 of the result through the tied output matrix."""
    W = {k: torch.zeros(s) for k, s in O.tensor_shapes(cfg).items()}
    W["embed"][:3, 0] = 1.0
    for t in range(3):
        W["embed"][t, 1 + t] = 1.0
    W["embed"][3, 5] = W["embed"][4, 6] = 1.0
    W["l0.ls1"].fill_(64.0)
    toks = [0 if i % 3 else 2 for i in range(T)]
    toks[far] = 1
    return W, toks


def _bf16(W):
    return {k: v.bfloat16() for k, v in W.items()}


def planted_attention(window: int, keep: int, far: int, T: int, heads=2,
                      dim=4):
    """A windowed attention with kept first tokens (its state-space side
    scaled to nothing) in which the ONE token with id 1 outscores all others
    by far and carries a value of its own: logit 3 is large where a row sees
    it, logit 4 where it does not. Returns (cfg, W, tokens)."""
    cfg = _bare("parallel", {
        "left": {"heads": heads, "kv_heads": 1, "dim": dim, "vdim": dim,
                 "scale": 24.0 / dim, "mask": {"size": window,
                                               "keep_first": keep}},
        "right": {"heads": 1, "vdim": 2, "state": 2, "groups": 1,
                  "norm_groups": 1, "conv": 2},
        "left_scale": 1.0, "right_scale": 0.0})
    W, toks = _planted(cfg, far, T)
    p = "l0.mix.left."
    W[p + "q"][::dim, 0] = 1.0          # every query points at axis 0
    W[p + "k"][0, 2] = 8.0              # only token 1's key has it
    W[p + "k"][1, 0] = 1.0
    W[p + "v"][0, 2] = 1.0              # value: axis 0 for token 1,
    W[p + "v"][1, 1] = W[p + "v"][1, 3] = 1.0    # axis 1 for the others
    W[p + "q.norm"].fill_(1.0)
    W[p + "k.norm"].fill_(1.0)
    W[p + "o"][5, ::dim] = 1.0
    W[p + "o"][6, 1::dim] = 1.0
    return cfg, _bf16(W), toks


def planted_latent(window: int, far: int, T: int, heads=2, dim=4, rank=4):
    """The same for a windowed latent attention."""
    cfg = _bare("latent_attention", {
        "heads": heads, "dim": dim, "vdim": dim, "kv_rank": rank,
        "scale": 12.0, "mask": {"size": window}})
    W, toks = _planted(cfg, far, T)
    p = "l0.mix."
    W[p + "q"][::dim, 0] = 2.0
    W[p + "dkv"][0, 2] = 2.0            # latent axis 0: token 1
    W[p + "dkv"][1, 1] = W[p + "dkv"][1, 3] = 2.0    # axis 1: the others
    W[p + "dkv.norm"].fill_(1.0)
    W[p + "uk"][::dim, 0] = 1.0
    W[p + "uv"][::dim, 0] = 1.0
    W[p + "uv"][1::dim, 1] = 1.0
    W[p + "g"][:, 0] = 4.0
    W[p + "o"][5, ::dim] = 1.0
    W[p + "o"][6, 1::dim] = 1.0
    return cfg, _bf16(W), toks


def planted_memory(far: int, T: int, taps=3):
    """A state-space recurrence (its attention side scaled to nothing) that
    forgets nothing and writes only for token id 1: logit 3 is large in every
    row from `far` on."""
    cfg = _bare("parallel", {
        "left": {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 2, "scale": 1.0,
                 "mask": {"size": 4, "keep_first": 1}},
        "right": {"heads": 1, "vdim": 2, "state": 3, "groups": 1,
                  "norm_groups": 1, "conv": taps},
        "left_scale": 0.0, "right_scale": 1.0})
    W, toks = _planted(cfg, far, T)
    p = "l0.mix.right."
    # rows: z 0-1, x 2-3, B 4-6, C 7-9, dt 10
    W[p + "in"][0:2, 0] = 4.0
    W[p + "in"][2, 2] = 4.0             # x: only token 1
    W[p + "in"][3, 0] = 4.0             # beside it a constant that only the
    W[p + "D"].fill_(1.0)               # skip carries, so the norm has a scale
    W[p + "in"][4, 2] = 4.0             # B likewise
    W[p + "in"][7, 0] = 4.0             # C: every row reads
    W[p + "conv"][:, -1] = 1.0
    W[p + "dt_bias"].fill_(1.0)
    W[p + "A_log"].fill_(-20.0)
    W[p + "norm"].fill_(1.0)
    W[p + "o"][5, 0] = 1.0
    for n in ("q.norm", "k.norm"):
        W["l0.mix.left." + n].fill_(1.0)
    return cfg, _bf16(W), toks
