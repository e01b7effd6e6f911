"""Small Nogapel configurations for the tests and weights that make faults show.

Random weights of one small scale would hide most faults: every softmax nearly uniform, every convolution close to
nothing, every gate half open.  ``make_weights`` draws bolder ones: head norms with weights away from one and latents large
enough for peaked attention, sinks that take a share of the softmax, convolutions whose earlier taps weigh as much as the
last, shares of mixed values between a quarter and three quarters, a token table that matters.  Everything is rounded to
bfloat16 once, so that both precisions run the same model.
"""

from __future__ import annotations

import math

import torch

from polosun_util import Fixed, make_runner, spread  # noqa: F401  (architecture-neutral helpers)

BANDS = {"factor": 5.0, "low": 0.5, "high": 3.0, "original": 64}

# every size differs from its neighbours'; the layer that mixes first is not the first layer, a layer between mixes
# nothing, and the mixing layers cut their value numbers differently; windows shorter than a page and longer, one layer
# without a feed-forward, latent attention with and without divided frequencies
SMALL_A = {
    "architecture": "Nogapel", "vocab": 96, "width": 64, "norm": {"eps": 1e-3}, "token_side": {"dim": 12},
    "layers": [
        {"type": "attention",
         "mixer": {"heads": 6, "kv_heads": 3, "dim": 16, "vdim": 20, "conv": 2, "scale": 0.3, "v_mix": False,
                   "mask": {"size": 21}, "rot": {"base": 100.0, "dims": 10}},
         "mlp": {"kind": "dense", "ff": 52}},
        {"type": "attention",
         "mixer": {"heads": 4, "kv_heads": 2, "dim": 24, "vdim": 12, "conv": 3, "scale": 0.25, "v_mix": True,
                   "mask": {"size": 9}, "rot": {"base": 1000.0, "dims": 24, "scaling": BANDS}},
         "mlp": {"kind": "dense", "ff": 72}},
        {"type": "latent_attention",
         "mixer": {"heads": 3, "dim": 16, "rot_dim": 8, "vdim": 24, "q_rank": 40, "kv_rank": 56, "scale": 0.3,
                   "rot": {"base": 1000.0, "dims": 8, "scaling": BANDS}},
         "mlp": {"kind": "dense", "ff": 80}},
        {"type": "attention",
         "mixer": {"heads": 3, "kv_heads": 1, "dim": 20, "vdim": 24, "conv": 4, "scale": 0.35, "v_mix": True,
                   "mask": {"size": 33}, "rot": {"base": 50.0, "dims": 8}},
         "mlp": None},
        {"type": "latent_attention",
         "mixer": {"heads": 5, "dim": 8, "rot_dim": 4, "vdim": 7, "q_rank": 16, "kv_rank": 24, "scale": 0.5,
                   "rot": {"base": 50.0, "dims": 4}},
         "mlp": {"kind": "dense", "ff": 40}},
        {"type": "attention",
         "mixer": {"heads": 3, "kv_heads": 3, "dim": 8, "vdim": 8, "conv": 3, "scale": 0.5, "v_mix": True,
                   "mask": {"size": 17}, "rot": {"base": 300.0, "dims": 4, "scaling": BANDS}},
         "mlp": {"kind": "dense", "ff": 33}},
    ],
}

# a width that is no multiple of 8, twenty query heads on one key head, six taps and one, windows of one token and longer
# than any test sequence, sizes of the latents that are no multiples of 8, an odd value size
SMALL_B = {
    "architecture": "Nogapel", "vocab": 130, "width": 50, "norm": {"eps": 2e-3}, "token_side": {"dim": 9},
    "layers": [
        {"type": "latent_attention",
         "mixer": {"heads": 20, "dim": 12, "rot_dim": 18, "vdim": 10, "q_rank": 33, "kv_rank": 150, "scale": 0.2,
                   "rot": {"base": 300.0, "dims": 18, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 2048}}},
         "mlp": {"kind": "dense", "ff": 44}},
        {"type": "attention",
         "mixer": {"heads": 20, "kv_heads": 1, "dim": 40, "vdim": 32, "conv": 6, "scale": 0.15, "v_mix": True,
                   "mask": {"size": 1000}, "rot": {"base": 10000.0, "dims": 40}},
         "mlp": None},
        {"type": "attention",
         "mixer": {"heads": 2, "kv_heads": 2, "dim": 136, "vdim": 16, "conv": 1, "scale": 0.1, "v_mix": True,
                   "mask": {"size": 7}, "rot": {"base": 30.0, "dims": 2}},
         "mlp": {"kind": "dense", "ff": 30}},
        {"type": "attention",
         "mixer": {"heads": 4, "kv_heads": 4, "dim": 10, "vdim": 9, "conv": 3, "scale": 0.4, "v_mix": False,
                   "mask": {"size": 1}, "rot": {"base": 30.0, "dims": 10, "scaling": BANDS}},
         "mlp": {"kind": "dense", "ff": 72}},
    ],
}

SMALL = {"A": SMALL_A, "B": SMALL_B}


def single(*layers: dict, width: int = 32, vocab: int = 50, side: int | None = 8) -> dict:
    """A model of one layer (or a few): a mechanism alone."""
    raw = {"architecture": "Nogapel", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "layers": list(layers)}
    if side is not None:
        raw["token_side"] = {"dim": side}
    return raw


def make_weights(raw: dict, seed: int) -> dict[str, torch.Tensor]:
    """Float32 tensors (bfloat16-representable values) for every name the configuration's model expects."""
    from cie_amd.config import config_from_dict
    from cie_amd.parts.model import expected_tensors

    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, spec in expected_tensors(config_from_dict(raw).model_spec()).items():
        shape = tuple(spec.random_shape)
        leaf = name.split(".", 1)[1] if name.startswith("l") and "." in name else name
        last = leaf.rsplit(".", 1)[-1]
        fan_in = shape[-1] if len(shape) >= 2 else 1
        normal = lambda scale: torch.randn(shape, generator=g) * scale
        if leaf in ("mix.q.norm", "mix.k.norm"):
            t = 0.8 + 0.9 * torch.rand(shape, generator=g)
        elif last in ("norm", "norm1"):
            t = 0.6 + 0.8 * torch.rand(shape, generator=g)
        elif last == "conv":
            t = normal(0.6)
        elif last == "vmix":
            t = 0.25 + 0.5 * torch.rand(shape, generator=g)
        elif last == "sink":
            t = normal(1.5)
        elif leaf in ("mix.uq", "mix.uk", "mix.dkv"):
            t = normal(1.4 / math.sqrt(fan_in))
        elif leaf == "side.gate":
            t = normal(1.5 / math.sqrt(fan_in))
        elif name in ("embed", "side.embed"):
            t = normal(1.0)
        else:
            t = normal(1.0 / math.sqrt(fan_in))
        out[name] = t
    return {name: t.to(torch.bfloat16).float() for name, t in out.items()}
