"""A plain, slow implementation of the Nogapel decoder, one function per mechanism, in float64 and without a cache.

It shares no code with the package: tests compare the engine with it.  A model is a raw configuration (the
``config.json`` dictionary) and a dictionary of tensors by checkpoint name.  Every function takes a whole sequence from
its first token (rows are tokens), so there is nothing to carry from step to step: what a token sees is said by a mask,
what a convolution reads by a shift.
"""

from __future__ import annotations

import math

import torch

F = torch.float64


# ---------------------------------------------------------------------------------------------------- mechanisms
def rms_norm(x: torch.Tensor, weight, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def squared_relu(z: torch.Tensor) -> torch.Tensor:
    return torch.where(z > 0, z * z, torch.zeros_like(z))


def short_convolution(u: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """u [tokens, channels], taps [channels, n]: the last tap meets the token itself, the one before it the token before."""
    n = taps.shape[1]
    y = torch.zeros_like(u)
    for back in range(n):
        if back < u.shape[0]:
            y[back:] += u[: u.shape[0] - back] * taps[:, n - 1 - back]
    return y


def frequencies(rot: dict) -> torch.Tensor:
    """Radians per position of every pair; with ``scaling``, waves longer than the length the base was made for turn
    ``factor`` times slower, short ones as they did, and those in between at a mean of the two."""
    out = []
    s = rot.get("scaling")
    for i in range(rot["dims"] // 2):
        f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
        if s is not None:
            turns = s["original"] * f / (2.0 * math.pi)      # how often the pair turns over that length
            if turns < s["low"]:
                f = f / s["factor"]
            elif turns <= s["high"]:
                keep = (turns - s["low"]) / (s["high"] - s["low"])
                f = f * keep + f / s["factor"] * (1.0 - keep)
        out.append(f)
    return torch.tensor(out, dtype=F)


def rotate(heads: torch.Tensor, rates: torch.Tensor) -> torch.Tensor:
    """heads [tokens, ..., dim]: numbers 2i and 2i + 1 turn together by the token's place times rate i; the rest stays."""
    n = 2 * rates.shape[0]
    place = torch.arange(heads.shape[0], dtype=F).reshape([-1] + [1] * (heads.dim() - 1))
    cos, sin = torch.cos(place * rates).to(heads.dtype), torch.sin(place * rates).to(heads.dtype)
    u, v = heads[..., 0:n:2], heads[..., 1:n:2]
    turned = torch.stack([u * cos - v * sin, v * cos + u * sin], dim=-1).flatten(-2)
    return torch.cat([turned, heads[..., n:]], dim=-1)


def mask(tokens: int, window=None) -> torch.Tensor:
    """[query, key]: itself and what came before it, at most ``window`` tokens in all."""
    back = torch.arange(tokens)[:, None] - torch.arange(tokens)[None, :]
    return (back >= 0) & (back < (window if window is not None else tokens))


def softmax(scores: torch.Tensor, seen: torch.Tensor, sink=None) -> torch.Tensor:
    """Over the last axis; ``sink`` is one more exponential in the denominator, which has no value."""
    scores = scores.masked_fill(~seen, -math.inf)
    top = scores.max(-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, sink)
    e = torch.exp(scores - top)
    total = e.sum(-1, keepdim=True)
    return e / (total if sink is None else total + torch.exp(sink - top))


def mix_values(own: torch.Tensor, first: torch.Tensor, share: torch.Tensor) -> torch.Tensor:
    return (1.0 - share) * own + share * first


def token_side(x: torch.Tensor, side_rows: torch.Tensor, gate: torch.Tensor, proj: torch.Tensor, weight: torch.Tensor,
               eps: float) -> torch.Tensor:
    """What a layer's own embedding of the tokens adds to the stream."""
    return rms_norm((gelu_tanh(x @ gate.t()) * side_rows) @ proj.t(), weight, eps)


# ---------------------------------------------------------------------------------------------------- the mixers
def attention(t: dict, p: str, c: dict, h: torch.Tensor, eps: float, carried: dict) -> torch.Tensor:
    tokens, heads, groups = h.shape[0], c["heads"], c.get("kv_heads", c["heads"])
    made = {}
    for name in ("q", "k", "v"):
        made[name] = h @ t[p + name].t()
        if c.get("conv") is not None:
            made[name] = short_convolution(made[name], t[f"{p}{name}.conv"])
    q, k = made["q"].reshape(tokens, heads, c["dim"]), made["k"].reshape(tokens, groups, c["dim"])
    q, k = rms_norm(q, t[p + "q.norm"], eps), rms_norm(k, t[p + "k.norm"], eps)
    if c.get("rot") is not None:
        rates = frequencies(c["rot"])
        q, k = rotate(q, rates), rotate(k, rates)
    v = made["v"]
    if c.get("v_mix"):
        if "first" not in carried:
            carried["first"] = v
        else:
            v = mix_values(v, carried["first"], t[p + "vmix"])
    v = v.reshape(tokens, groups, c["vdim"])
    seen = mask(tokens, (c.get("mask") or {}).get("size"))
    outs = []
    for i in range(heads):
        g = i // (heads // groups)
        outs.append(softmax(q[:, i] @ k[:, g].t() * float(c["scale"]), seen) @ v[:, g])
    return torch.cat(outs, -1) @ t[p + "o"].t()


def latent_attention(t: dict, p: str, c: dict, h: torch.Tensor, eps: float, carried: dict) -> torch.Tensor:
    tokens, heads, dim, turned, rank = h.shape[0], c["heads"], c["dim"], c["rot_dim"], c["kv_rank"]
    rates = frequencies(c["rot"])
    q = (rms_norm(h @ t[p + "dq"].t(), t[p + "dq.norm"], eps) @ t[p + "uq"].t()).reshape(tokens, heads, dim + turned)
    down = h @ t[p + "dkv"].t()
    latent = rms_norm(down[:, :rank], t[p + "dkv.norm"], eps)
    shared = rotate(down[:, rank:], rates)
    plain_k = (latent @ t[p + "uk"].t()).reshape(tokens, heads, dim)
    v = (latent @ t[p + "uv"].t()).reshape(tokens, heads, c["vdim"])
    q_turned = rotate(q[..., dim:], rates)
    seen = mask(tokens, (c.get("mask") or {}).get("size"))
    outs = []
    for i in range(heads):
        scores = (q[:, i, :dim] @ plain_k[:, i].t() + q_turned[:, i] @ shared.t()) * float(c["scale"])
        outs.append(softmax(scores, seen, t[p + "sink"][i]) @ v[:, i])
    return torch.cat(outs, -1) @ t[p + "o"].t()


def feed_forward(t: dict, p: str, h: torch.Tensor) -> torch.Tensor:
    return squared_relu(h @ t[p + "up"].t()) @ t[p + "down"].t()


# ---------------------------------------------------------------------------------------------------- the model
MIXERS = {"attention": attention, "latent_attention": latent_attention}


class Model:
    """``dtype``: float64 is the yardstick; bfloat16 shows what rounding everything to 16 bits costs."""

    def __init__(self, config: dict, tensors: dict, dtype: torch.dtype = F) -> None:
        self.config = config
        self.t = {name: value.to(dtype) for name, value in tensors.items()}
        self.eps = float(config["norm"]["eps"])

    def streams(self, tokens) -> list[torch.Tensor]:
        """The stream as the embedding makes it, and after every layer."""
        t, ids = self.t, torch.as_tensor(list(tokens), dtype=torch.long)
        x = rms_norm(t["embed"][ids], t["embed.norm"], self.eps)
        side = self.config.get("token_side")
        out, carried = [x], {}
        for i, layer in enumerate(self.config["layers"]):
            p = f"l{i}."
            h = rms_norm(x, t[p + "norm1"], self.eps)
            branch = MIXERS[layer["type"]](t, p + "mix.", layer["mixer"], h, self.eps, carried)
            if layer.get("mlp") is not None:
                branch = branch + feed_forward(t, p + "mlp.", h)
            x = x + branch
            if side is not None:
                rows = t["side.embed"][ids][:, i * side["dim"]: (i + 1) * side["dim"]]
                x = x + token_side(x, rows, t[p + "side.gate"], t[p + "side.proj"], t[p + "side.norm"], self.eps)
            out.append(x)
        return out

    def logits(self, tokens) -> torch.Tensor:
        return rms_norm(self.streams(tokens)[-1], self.t["final.norm"], self.eps) @ self.t["head"].t()


def forward(config: dict, tensors: dict, tokens, dtype: torch.dtype = F) -> torch.Tensor:
    """Logits [len(tokens), vocab] of one sequence from its start."""
    return Model(config, tensors, dtype).logits(tokens)
