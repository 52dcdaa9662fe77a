"""Helpers of the Tudatar tests: write a small random checkpoint, serve it
with the engine; replay/compare helpers are shared with the other hybrid
families' tests."""
from __future__ import annotations

from typing import Sequence

import torch

from tests import tudatar_oracle as O
from tests.nukopel_util import (assert_logits, chunk_schedule,  # noqa: F401
                                random_tokens, rel_err, replay, row_errs)


def make_engine(tmp_path, cfg, W, device="cpu", dtype=torch.float32,
                max_batch=4, block_size=16, kv_blocks=64, max_seq_len=1024,
                **kw):
    from bee2bee_amd.engine.engine import InferenceEngine

    path = str(tmp_path / "ckpt")
    O.save_checkpoint(path, cfg, W)
    return InferenceEngine(
        "td-test", device=device, dtype=dtype, model_path=path,
        max_batch=max_batch, max_seq_len=max_seq_len,
        use_graphs=kw.pop("use_graphs", False), kv_block_size=block_size,
        kv_blocks=kv_blocks, kv_margin_blocks=1, **kw)


def oracle_logits(cfg, W, tokens: Sequence[int]) -> torch.Tensor:
    return O.forward(cfg, W, list(tokens))


def single_mixer(kind: str, mixer: dict, width: int, vocab: int) -> dict:
    """A config with one layer of one mixer and no feed-forward."""
    return {"architecture": "Tudatar", "vocab": vocab, "width": width,
            "norm": {"eps": 1e-5}, "logit_scale": 1.0,
            "layers": [{"type": kind, "mixer": mixer, "mlp": None}]}


def plain_norms(W, width: int, names: Sequence[str], alpha=0.0625) -> None:
    """Norms near the identity for small inputs: tanh(a x) / a."""
    for n in names:
        W[n] = torch.full((width,), 1.0 / alpha).bfloat16()
        W[n + ".b"] = torch.zeros(width).bfloat16()
        W[n + ".alpha"] = torch.tensor(alpha).bfloat16()


def planted_attention(window: int, far: int, T: int, heads=2, dim=4):
    """One windowed attention layer over one-hot-like token vectors in which
    ONE token (id 1, placed at `far`) outscores all others by far and
    carries a value of its own; every other token is id 0 or 2. Returns
    (cfg, W, tokens)."""
    width, vocab = 8, 3
    cfg = single_mixer("attention", {
        "heads": heads, "kv_heads": 1, "dim": dim, "vdim": dim, "scale": 6.0,
        "mask": {"size": window}}, width, vocab)
    W = {k: torch.zeros(s) for k, s in O.tensor_shapes(cfg).items()}
    # x: [one, is0, is1, is2, 0...]
    W["embed"][:, 0] = 1.0
    for t in range(3):
        W["embed"][t, 1 + t] = 1.0
    p = "l0.mix."
    W[p + "q"][::dim, 0] = 1.0               # every query points at axis 0
    W[p + "k"][0, 2] = 4.0                   # only token 1's key has it
    W[p + "k"][1, 0] = 1.0
    W[p + "v"][0, 2] = 1.0                   # value: axis 0 for token 1,
    W[p + "v"][1, 1] = W[p + "v"][1, 3] = 1.0    # axis 1 for the others
    W[p + "q.norm"].fill_(1.0)
    W[p + "k.norm"].fill_(1.0)
    W[p + "r1"].fill_(0.125)
    W[p + "r2"].fill_(1.0)
    W[p + "o"][5, ::dim] = 1.0               # axis 0 of the heads -> x[5]
    W[p + "o"][6, 1::dim] = 1.0
    W["head"][0, 5] = W["head"][1, 6] = W["head"][2, 0] = 1.0
    plain_norms(W, width, ("l0.norm1", "l0.norm1b", "final.norm"))
    W = {k: v.bfloat16() for k, v in W.items()}
    toks = [0 if i % 3 else 2 for i in range(T)]
    toks[far] = 1
    return cfg, W, toks
