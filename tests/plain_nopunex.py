"""A plain, slow implementation of the Nopunex decoder, one function per mechanism, in float64 and token by token.

It shares no code with the package: tests compare the engine with it.  A model is a raw configuration (the
``config.json`` dictionary) and a dictionary of tensors by checkpoint name.  ``Model.start()`` gives a ``Sequence``
that is fed tokens one at a time (or in runs) and keeps, for every run of a layer separately, what the design carries
from token to token: keys and values, latents and turned key parts, the delta rule's memories and the convolutions'
last inputs.
"""

from __future__ import annotations

import math

import torch

F = torch.float64


# ---------------------------------------------------------------------------------------------------- mechanisms
def layer_norm(x: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor, eps: float) -> torch.Tensor:
    centred = x - x.mean(-1, keepdim=True)
    return centred / torch.sqrt((centred * centred).mean(-1, keepdim=True) + eps) * weight + bias


def rms_norm(x: torch.Tensor, weight, eps: float) -> torch.Tensor:
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.log1p(torch.exp(-z.abs())) + z.clamp(min=0.0)


def unit(x: torch.Tensor) -> torch.Tensor:
    """x at length one (a row of zeros stays one)."""
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def frequencies(rot: dict) -> tuple[torch.Tensor, float]:
    """The turning rates of the pairs, and the factor on cos and sin."""
    dims, base = rot["dims"], float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if s is None:
        return torch.tensor(f, dtype=F), 1.0
    at = lambda turns: dims * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(at(s["fast"])), 0), min(math.ceil(at(s["slow"])), dims - 1)
    ramp = [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(dims // 2)]
    return (torch.tensor([fi / s["factor"] * r + fi * (1.0 - r) for fi, r in zip(f, ramp)], dtype=F),
            0.1 * math.log(s["factor"]) + 1.0)


def rotate(heads: torch.Tensor, position: int, rates: torch.Tensor, gain: float) -> torch.Tensor:
    """Turn the first numbers of every head, number i together with number i + dims / 2."""
    half = rates.shape[0]
    cos = (torch.cos(position * rates) * gain).to(heads.dtype)
    sin = (torch.sin(position * rates) * gain).to(heads.dtype)
    u, v, rest = heads[..., :half], heads[..., half: 2 * half], heads[..., 2 * half:]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, rest], dim=-1)


def window_sees(i: int, j: int, size) -> bool:
    return j <= i and (size is None or i - j < size)


def chunk_sees(i: int, j: int, size) -> bool:
    return j <= i and (size is None or i // size == j // size)


def softmax_weights(scores: torch.Tensor, sink=None) -> torch.Tensor:
    """Softmax over the last axis; ``sink`` is one more score in the denominator that has no value."""
    top = scores.max() if sink is None else torch.maximum(scores.max(), sink)
    e = torch.exp(scores - top)
    return e / (e.sum() + (torch.exp(sink - top) if sink is not None else 0.0))


def differential(first: torch.Tensor, second: torch.Tensor, lam, diff: float, eps: float) -> torch.Tensor:
    """Two maps' outputs over the same values to one head's output."""
    return rms_norm(first - lam * second, None, eps) * (1.0 - diff)


def delta_token(memory: torch.Tensor, q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, beta: torch.Tensor,
                decay: torch.Tensor) -> tuple[torch.Tensor, torch.Tensor]:
    """One head, memory [dim, vdim]: it fades, is corrected towards v at k, and is read at q."""
    memory = decay * memory
    u = beta * (v - memory.t() @ k)
    memory = memory + torch.outer(k, u)
    return memory, memory.t() @ q


# ---------------------------------------------------------------------------------------------------- the model
class Model:
    def __init__(self, config: dict, tensors: dict, dtype: torch.dtype = F) -> None:
        self.config = config
        self.dtype = dtype  # float64 is the yardstick; bfloat16 shows what rounding everything to 16 bits costs
        self.t = {name: value.to(dtype) for name, value in tensors.items()}
        self.eps = float(config["norm"]["eps"])
        self.layers = config["layers"]
        loop = config.get("loop") or {"start": 0, "stop": 0, "times": 0}
        start, stop = loop["start"], loop["stop"]
        # the runs in order: (layer, number of the pass that begins with it, or None)
        self.runs = [(i, None) for i in range(start)]
        for turn in range(loop["times"] if stop > start else 0):
            self.runs += [(i, turn if i == start else None) for i in range(start, stop)]
        self.runs += [(i, None) for i in range(stop, len(self.layers))]

    def start(self) -> "Sequence":
        return Sequence(self)

    def logits(self, tokens) -> torch.Tensor:
        """Logits [len(tokens), vocab] of one sequence from its start."""
        return self.start().feed(tokens)


class Sequence:
    def __init__(self, model: Model) -> None:
        self.m = model
        self.position = 0
        self.kept: dict[tuple, list] = {}             # (run, what) -> one entry per token
        self.state: dict[tuple, torch.Tensor] = {}    # (run, what) -> tensor
        self.stream_after: list[list[torch.Tensor]] = []  # per token, the stream after every run of a layer

    def feed(self, tokens) -> torch.Tensor:
        return torch.stack([self.token(int(t)) for t in tokens])

    def norm(self, name: str, x: torch.Tensor) -> torch.Tensor:
        return layer_norm(x, self.m.t[name], self.m.t[name + ".b"], self.m.eps)

    def token(self, token: int) -> torch.Tensor:
        m, t = self.m, self.m.t
        embedded = t["embed"][token].clone()
        x = embedded
        after = []
        for run, (index, turn) in enumerate(m.runs):
            layer, p = m.layers[index], f"l{index}."
            if turn is not None:
                x = t["loop.in"] @ torch.cat([x, embedded]) + t["loop.step"][turn]
            mixer = {"delta": self.delta, "latent_attention": self.latent_attention, "attention": self.attention}[layer["type"]]
            x = x + self.norm(p + "norm1b", mixer(run, layer["mixer"], p + "mix.", self.norm(p + "norm1", x)))
            if layer.get("mlp") is not None:
                x = x + self.norm(p + "norm2b", self.feed_forward(p + "mlp.", self.norm(p + "norm2", x)))
            after.append(x.clone())
        self.stream_after.append(after)
        self.position += 1
        return t["head"] @ self.norm("final.norm", x) * float(m.config.get("logit_scale", 1.0))

    # -- the gated delta rule
    def short_convolution(self, run: int, name: str, x: torch.Tensor) -> torch.Tensor:
        weight = self.m.t[name + ".conv"]                                      # [channels, taps]
        past = self.state.get((run, name), torch.zeros((weight.shape[1] - 1, x.shape[0]), dtype=x.dtype))
        inputs = torch.cat([past, x[None]], dim=0)                              # oldest first
        self.state[(run, name)] = inputs[1:]
        return silu((inputs * weight.t()).sum(0))

    def delta(self, run: int, c: dict, p: str, h: torch.Tensor) -> torch.Tensor:
        m, t = self.m, self.m.t
        heads, shared, dim, vdim = c["heads"], c.get("kv_heads", c["heads"]), c["dim"], c["vdim"]
        q = unit(self.short_convolution(run, p + "q", t[p + "q"] @ h).reshape(shared, dim)) * dim ** -0.5
        k = unit(self.short_convolution(run, p + "k", t[p + "k"] @ h).reshape(shared, dim))
        v = self.short_convolution(run, p + "v", t[p + "v"] @ h).reshape(heads, vdim)
        beta = torch.sigmoid(t[p + "b"] @ h)
        decay = torch.exp(-torch.exp(t[p + "A_log"]) * softplus(t[p + "a"] @ h + t[p + "dt_bias"]))
        gate = silu(t[p + "g"] @ h).reshape(heads, vdim)
        memory = self.state.get((run, "memory"), torch.zeros((heads, dim, vdim), dtype=m.dtype))
        new, outs = [], []
        for i in range(heads):
            j = i // (heads // shared)
            s, o = delta_token(memory[i], q[j], k[j], v[i], beta[i], decay[i])
            new.append(s)
            outs.append(rms_norm(o, t[p + "norm"], m.eps) * gate[i])
        self.state[(run, "memory")] = torch.stack(new)
        return t[p + "o"] @ torch.cat(outs)

    # -- latent attention under a window with a sink
    def latent_attention(self, run: int, c: dict, p: str, h: torch.Tensor) -> torch.Tensor:
        m, t = self.m, self.m.t
        heads, dim, turned, vdim, rank = c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
        rates, gain = frequencies(c["rot"])
        q = (t[p + "uq"] @ rms_norm(t[p + "dq"] @ h, t[p + "dq.norm"], m.eps)).reshape(heads, dim + turned)
        down = t[p + "dkv"] @ h
        latents = self.kept.setdefault((run, "latent"), [])
        keys = self.kept.setdefault((run, "key"), [])
        latents.append(rms_norm(down[:rank], t[p + "dkv.norm"], m.eps))
        keys.append(rotate(down[rank:], self.position, rates, gain))
        seen = [j for j in range(self.position + 1) if window_sees(self.position, j, (c.get("mask") or {}).get("size"))]
        all_c = torch.stack([latents[j] for j in seen])
        all_k = torch.stack([keys[j] for j in seen])
        uk, uv = t[p + "uk"].reshape(heads, dim, rank), t[p + "uv"].reshape(heads, vdim, rank)
        outs = []
        for i in range(heads):
            scores = ((all_c @ uk[i].t()) @ q[i, :dim] + all_k @ rotate(q[i, dim:], self.position, rates, gain)) * float(c["scale"])
            outs.append(softmax_weights(scores, t[p + "sink"][i]) @ (all_c @ uv[i].t()))
        return t[p + "o"] @ torch.cat(outs)

    # -- differential attention in chunks with a gate on its output
    def attention(self, run: int, c: dict, p: str, h: torch.Tensor) -> torch.Tensor:
        m, t = self.m, self.m.t
        heads, groups, dim, vdim = c["heads"], c.get("kv_heads", c["heads"]), c["dim"], c["vdim"]
        q, k = (t[p + "q"] @ h).reshape(heads, 2, dim), (t[p + "k"] @ h).reshape(groups, 2, dim)
        if c.get("rot") is not None:
            rates, gain = frequencies(c["rot"])
            q, k = rotate(q, self.position, rates, gain), rotate(k, self.position, rates, gain)
        keys, values = self.kept.setdefault((run, "key"), []), self.kept.setdefault((run, "value"), [])
        keys.append(k)
        values.append((t[p + "v"] @ h).reshape(groups, vdim))
        seen = [j for j in range(self.position + 1) if chunk_sees(self.position, j, (c.get("mask") or {}).get("size"))]
        all_k, all_v = torch.stack([keys[j] for j in seen]), torch.stack([values[j] for j in seen])
        lam = (torch.exp((t[p + "lq1"] * t[p + "lk1"]).sum()) - torch.exp((t[p + "lq2"] * t[p + "lk2"]).sum())
               + float(c["diff"]))
        outs = []
        for i in range(heads):
            g = i // (heads // groups)
            maps = [softmax_weights((all_k[:, g, n] @ q[i, n]) * float(c["scale"])) @ all_v[:, g] for n in range(2)]
            outs.append(differential(maps[0], maps[1], lam, float(c["diff"]), m.eps))
        return t[p + "o"] @ (torch.cat(outs) * torch.sigmoid(t[p + "g"] @ h))

    def feed_forward(self, p: str, h: torch.Tensor) -> torch.Tensor:
        t = self.m.t
        return t[p + "down"] @ (silu(t[p + "gate"] @ h) * (t[p + "up"] @ h))


def forward(config: dict, tensors: dict, tokens, dtype: torch.dtype = F) -> torch.Tensor:
    """Logits [len(tokens), vocab] of one sequence from its start."""
    return Model(config, tensors, dtype).logits(tokens)
