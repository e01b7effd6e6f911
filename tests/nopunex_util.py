"""Small Nopunex configurations for the tests and weights that make faults show.

Random weights of one small scale would hide most faults: every softmax nearly uniform, every step size one half, every
decay the same, every difference of two maps zero.  ``make_weights`` draws bolder ones: queries and keys large enough for
peaked attention, sinks that take a share of the softmax, step sizes and decays spread over their range, gates that open
and close, norm weights away from one and biases away from zero, steps of the passes that differ.  Everything is rounded
to bfloat16 once, so that both precisions run the same model.
"""

from __future__ import annotations

import math

import torch

from polosun_util import Fixed, make_runner, spread  # noqa: F401  (architecture-neutral helpers)

YARN = {"factor": 4.0, "fast": 16.0, "original": 64, "slow": 1.0}

# every size differs from its neighbours'; a delta layer with shared key heads and one with a feed-forward, one tap and
# a key head for every head; latent attention with and without a stretch and a window; a run of two layers that passes
# three times
SMALL_A = {
    "architecture": "Nopunex", "vocab": 96, "width": 64, "norm": {"eps": 1e-3}, "logit_scale": 1.5,
    "loop": {"start": 1, "stop": 3, "times": 3},
    "layers": [
        {"type": "delta", "mixer": {"heads": 4, "kv_heads": 2, "dim": 12, "vdim": 20, "conv": 3}, "mlp": None},
        {"type": "latent_attention",
         "mixer": {"heads": 3, "dim": 16, "rot_dim": 8, "vdim": 24, "q_rank": 40, "kv_rank": 56, "scale": 0.3,
                   "mask": {"size": 9}, "rot": {"base": 1000.0, "dims": 8, "scaling": YARN}},
         "mlp": {"kind": "dense", "ff": 72}},
        {"type": "attention",
         "mixer": {"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 12, "scale": 0.35, "diff": 0.3, "mask": {"size": 11},
                   "rot": {"base": 100.0, "dims": 8}},
         "mlp": {"kind": "dense", "ff": 80}},
        {"type": "delta", "mixer": {"heads": 3, "kv_heads": 3, "dim": 20, "vdim": 8, "conv": 1},
         "mlp": {"kind": "dense", "ff": 56}},
        {"type": "latent_attention",
         "mixer": {"heads": 5, "dim": 8, "rot_dim": 4, "vdim": 8, "q_rank": 16, "kv_rank": 24, "scale": 0.5,
                   "rot": {"base": 50.0, "dims": 4}},
         "mlp": None},
    ],
}

# a width that is no multiple of 8, twenty query heads on one key head, a latent entry wider than most matrix-core forms
# take, chunks longer than any test sequence, the whole model passing twice with the attention first, sizes of the
# latents that are no multiples of 8, five taps
SMALL_B = {
    "architecture": "Nopunex", "vocab": 130, "width": 50, "norm": {"eps": 2e-3}, "logit_scale": 0.75,
    "loop": {"start": 0, "stop": 4, "times": 2},
    "layers": [
        {"type": "attention",
         "mixer": {"heads": 20, "kv_heads": 1, "dim": 40, "vdim": 32, "scale": 0.1, "diff": 0.8, "mask": {"size": 1000},
                   "rot": {"base": 10000.0, "dims": 40}},
         "mlp": None},
        {"type": "latent_attention",
         "mixer": {"heads": 20, "dim": 12, "rot_dim": 18, "vdim": 10, "q_rank": 33, "kv_rank": 150, "scale": 0.2,
                   "mask": {"size": 33}, "rot": {"base": 300.0, "dims": 18, "scaling": {"factor": 8.0, "fast": 32.0, "original": 2048, "slow": 1.0}}},
         "mlp": {"kind": "dense", "ff": 72}},
        {"type": "delta", "mixer": {"heads": 5, "kv_heads": 1, "dim": 72, "vdim": 24, "conv": 5},
         "mlp": {"kind": "dense", "ff": 44}},
        {"type": "attention",
         "mixer": {"heads": 2, "kv_heads": 2, "dim": 136, "vdim": 8, "scale": 0.05, "diff": 0.1, "mask": {"size": 7},
                   "rot": {"base": 30.0, "dims": 2}},
         "mlp": {"kind": "dense", "ff": 30}},
    ],
}

SMALL = {"A": SMALL_A, "B": SMALL_B}


def single(layer: dict, width: int = 32, vocab: int = 50, loop: dict | None = None) -> dict:
    """A model of one layer: a mechanism alone (``loop``: passing several times)."""
    raw = {"architecture": "Nopunex", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "logit_scale": 1.0, "layers": [layer]}
    if loop is not None:
        raw["loop"] = loop
    return raw


def make_weights(raw: dict, seed: int) -> dict[str, torch.Tensor]:
    """Float32 tensors (bfloat16-representable values) for every name the configuration's model expects."""
    from cie_amd.config import config_from_dict
    from cie_amd.parts.model import expected_tensors

    expected = expected_tensors(config_from_dict(raw).model_spec())
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, spec in expected.items():
        if spec.optional:
            continue
        shape = tuple(spec.random_shape)
        leaf = name.split(".", 1)[1] if name.startswith("l") and "." in name else name
        last = leaf.rsplit(".", 1)[-1]
        fan_in = shape[-1] if len(shape) >= 2 else 1
        normal = lambda scale: torch.randn(shape, generator=g) * scale
        if name == "loop.in":
            t = normal(0.7 / math.sqrt(fan_in))
        elif name == "loop.step":
            t = normal(0.5)
        elif leaf in ("norm1", "norm2", "norm1b", "norm2b") or name == "final.norm" or leaf.endswith(".norm"):
            t = 0.6 + 0.8 * torch.rand(shape, generator=g)
        elif leaf.endswith(".b") and leaf != "mix.b":                    # biases of the norms
            t = normal(0.3)
        elif last == "conv":
            t = normal(0.6)
        elif leaf in ("mix.q", "mix.k", "mix.uq", "mix.uk", "mix.dkv", "mix.b", "mix.a"):
            t = normal(1.4 / math.sqrt(fan_in))
        elif leaf == "mix.g":
            t = normal(2.0 / math.sqrt(fan_in))
        elif last == "sink":
            t = normal(1.5)
        elif last in ("lq1", "lk1", "lq2", "lk2"):
            t = normal(0.8 / math.sqrt(shape[0]) ** 0.5)
        elif leaf == "mix.A_log":
            t = torch.linspace(-2.0, 1.0, shape[0])[torch.randperm(shape[0], generator=g)]
        elif leaf == "mix.dt_bias":
            t = torch.linspace(-4.0, 0.5, shape[0])[torch.randperm(shape[0], generator=g)]
        elif name == "embed":
            t = normal(1.0)
        elif last in ("gate", "up"):
            t = normal(1.5 / math.sqrt(fan_in))
        else:
            t = normal(1.0 / math.sqrt(fan_in))
        out[name] = t
    return {name: t.to(torch.bfloat16).float() for name, t in out.items()}
