"""CPU: what pins the plain Nopunex implementation (tests/plain_nopunex.py), and the configuration's reading, which needs
no GPU."""

from __future__ import annotations

import copy
import math

import pytest
import torch

import nopunex_util as nu
import plain_nopunex as pn

F = torch.float64


def test_layer_norm_against_the_library():
    x, w, b = torch.randn(5, 12, dtype=F) * 3 + 2, torch.rand(12, dtype=F) + 0.5, torch.randn(12, dtype=F)
    want = torch.nn.functional.layer_norm(x, (12,), w, b, 1e-3)
    assert torch.allclose(pn.layer_norm(x, w, b, 1e-3), want, rtol=1e-12, atol=1e-13)


def test_rotation_by_halves_is_a_complex_multiplication():
    head = torch.randn(3, 12, dtype=F)
    rates, gain = pn.frequencies({"dims": 8, "base": 100.0})
    assert gain == 1.0
    turned = pn.rotate(head, 7, rates, gain)
    z = torch.complex(head[:, :4], head[:, 4:8]) * torch.polar(torch.ones(4, dtype=F), 7 * rates)
    assert torch.allclose(turned[:, :4], z.real, rtol=1e-13, atol=1e-14) and torch.allclose(turned[:, 4:8], z.imag, rtol=1e-13, atol=1e-14)
    assert torch.equal(turned[:, 8:], head[:, 8:])
    # scores depend on the distance alone
    a, b = torch.randn(8, dtype=F), torch.randn(8, dtype=F)
    assert torch.allclose(pn.rotate(a, 9, rates, 1.0) @ pn.rotate(b, 4, rates, 1.0), pn.rotate(a, 105, rates, 1.0) @ pn.rotate(b, 100, rates, 1.0), rtol=1e-9)


def test_stretched_frequencies_against_the_package_tables():
    from cie_amd.parts.position import RotaryHalf

    for rot in ({"dims": 8, "base": 1000.0, "scaling": nu.YARN},
                {"dims": 18, "base": 300.0, "scaling": {"factor": 8.0, "fast": 32.0, "original": 2048, "slow": 1.0}}):
        rates, gain = pn.frequencies(rot)
        s = rot["scaling"]
        got, g = RotaryHalf(20, rot["base"], None, rotary_dim=rot["dims"], scaling=(s["factor"], s["original"], s["fast"], s["slow"])).inv_freq()
        assert abs(g - gain) < 1e-12 and abs(gain - (0.1 * math.log(s["factor"]) + 1.0)) < 1e-12
        assert torch.allclose(got.double(), rates, rtol=1e-5)
    plain, _ = pn.frequencies({"dims": 8, "base": 1000.0})
    rates, _ = pn.frequencies({"dims": 8, "base": 1000.0, "scaling": nu.YARN})
    assert torch.allclose(rates[0], plain[0]) and torch.allclose(rates[-1], plain[-1] / 4.0)


def test_window_and_chunk_masks():
    assert pn.window_sees(20, 16, 5) and not pn.window_sees(20, 15, 5) and not pn.window_sees(20, 21, 5) and pn.window_sees(20, 0, None)
    assert pn.window_sees(3, 3, 1) and not pn.window_sees(3, 2, 1)
    assert pn.chunk_sees(12, 10, 5) and not pn.chunk_sees(12, 9, 5) and pn.chunk_sees(9, 5, 5) and not pn.chunk_sees(9, 10, 5)
    assert pn.chunk_sees(10, 10, 5) and not pn.chunk_sees(10, 9, 5) and pn.chunk_sees(99, 0, None)


def test_the_sink_is_one_more_column_of_the_softmax():
    scores, sink = torch.randn(7, dtype=F), torch.tensor(0.7, dtype=F)
    want = torch.softmax(torch.cat([scores, sink[None]]), 0)[:7]
    assert torch.allclose(pn.softmax_weights(scores, sink), want, rtol=1e-13)
    assert torch.allclose(pn.softmax_weights(scores), torch.softmax(scores, 0), rtol=1e-13)


def test_the_difference_of_two_maps_is_normed_without_a_weight():
    a, b = torch.randn(6, dtype=F), torch.randn(6, dtype=F)
    d = a - 0.4 * b
    assert torch.allclose(pn.differential(a, b, 0.4, 0.3, 1e-2), d / torch.sqrt((d ** 2).sum() / 6 + 1e-2) * 0.7, rtol=1e-13)


def test_the_delta_rule_against_its_definition_and_what_it_promises():
    """The update written out (the read-out sees the token's own write); with a step size of one and no decay the
    memory answers with exactly what was written last under a key, whatever lay there before."""
    n, N, P = 9, 5, 4
    q, k, v = torch.randn(n, N, dtype=F), pn.unit(torch.randn(n, N, dtype=F)), torch.randn(n, P, dtype=F)
    beta, decay = torch.rand(n, dtype=F), torch.rand(n, dtype=F)
    memory = S = torch.zeros(N, P, dtype=F)
    eye = torch.eye(N, dtype=F)
    for t in range(n):
        memory, o = pn.delta_token(memory, q[t], k[t], v[t], beta[t], decay[t])
        S = decay[t] * (eye - beta[t] * torch.outer(k[t], k[t])) @ S + beta[t] * torch.outer(k[t], v[t])
        assert torch.allclose(memory, S, rtol=1e-11, atol=1e-13) and torch.allclose(o, q[t] @ S, rtol=1e-11, atol=1e-13)
    one = torch.tensor(1.0, dtype=F)
    key = torch.zeros(N, dtype=F)
    key[2] = 1.0
    memory, o = pn.delta_token(memory, key, key, v[0], one, one)
    assert torch.allclose(o, v[0], rtol=1e-12)
    memory, o = pn.delta_token(memory, key, key, v[1], one, one)
    assert torch.allclose(o, v[1], rtol=1e-12)


def test_the_short_convolution_is_the_librarys():
    raw = nu.single({"type": "delta", "mixer": {"heads": 2, "kv_heads": 1, "dim": 4, "vdim": 3, "conv": 3}, "mlp": None})
    w = {k: v.double() for k, v in nu.make_weights(raw, seed=1).items()}
    seq = pn.Model(raw, w).start()
    x = torch.randn(7, 4, dtype=F)
    got = torch.stack([seq.short_convolution(0, "l0.mix.q", row) for row in x])
    padded = torch.cat([torch.zeros(2, 4, dtype=F), x]).t()[None]
    want = torch.nn.functional.silu(torch.nn.functional.conv1d(padded, w["l0.mix.q.conv"][:, None, :], groups=4))[0].t()
    assert torch.allclose(got, want, rtol=1e-12, atol=1e-14)


def test_a_model_composed_by_hand():
    """The first token of a model of one attention layer that passes twice: the joining product in front of each pass,
    norms on both sides, one key (every softmax is one), the scale on the logits."""
    layer = copy.deepcopy(nu.SMALL_A["layers"][2])
    raw = nu.single(layer, width=40, loop={"start": 0, "stop": 1, "times": 2})
    raw["logit_scale"] = 3.0
    w = {k: v.double() for k, v in nu.make_weights(raw, seed=1).items()}
    logits = pn.forward(raw, w, [3])[0]
    ln = lambda n, x: torch.nn.functional.layer_norm(x, (40,), w[n], w[n + ".b"], 1e-6)
    lam = math.exp(float(w["l0.mix.lq1"] @ w["l0.mix.lk1"])) - math.exp(float(w["l0.mix.lq2"] @ w["l0.mix.lk2"])) + 0.3
    x0 = x = w["embed"][3]
    for turn in range(2):
        x = w["loop.in"] @ torch.cat([x, x0]) + w["loop.step"][turn]
        h = ln("l0.norm1", x)
        v = (w["l0.mix.v"] @ h).reshape(2, 12).repeat_interleave(2, 0) * (1.0 - lam)
        v = v / torch.sqrt((v ** 2).mean(1, keepdim=True) + 1e-6) * 0.7
        x = x + ln("l0.norm1b", w["l0.mix.o"] @ (v.reshape(-1) * torch.sigmoid(w["l0.mix.g"] @ h)))
        h = ln("l0.norm2", x)
        x = x + ln("l0.norm2b", w["l0.mlp.down"] @ (torch.nn.functional.silu(w["l0.mlp.gate"] @ h) * (w["l0.mlp.up"] @ h)))
    assert torch.allclose(logits, 3.0 * (w["head"] @ ln("final.norm", x)), rtol=1e-10, atol=1e-12)


def test_latent_attention_against_library_attention_on_expanded_keys():
    raw = nu.single(copy.deepcopy(nu.SMALL_A["layers"][1]), width=64)
    raw["layers"][0]["mlp"] = None
    w = {k: v.double() for k, v in nu.make_weights(raw, seed=2).items()}
    c, p, n = raw["layers"][0]["mixer"], "l0.mix.", 20
    h = torch.randn(n, 64, dtype=F)
    seq = pn.Model(raw, w).start()
    got = []
    for t in range(n):
        got.append(seq.latent_attention(0, c, p, h[t]))
        seq.position += 1
    rates, gain = pn.frequencies(c["rot"])
    rms = lambda x, g: torch.nn.functional.rms_norm(x, (x.shape[-1],), g, 1e-6)
    q = (rms(h @ w[p + "dq"].t(), w[p + "dq.norm"]) @ w[p + "uq"].t()).reshape(n, 3, 24)
    down = h @ w[p + "dkv"].t()
    lat = rms(down[:, :56], w[p + "dkv.norm"])
    turn = lambda x, t: pn.rotate(x, t, rates, gain)
    q = torch.stack([torch.cat([q[t, :, :16], turn(q[t, :, 16:], t)], -1) for t in range(n)])
    k = torch.stack([torch.cat([(w[p + "uk"] @ lat[t]).reshape(3, 16), turn(down[t, 56:], t).expand(3, 8)], -1) for t in range(n)])
    v = (lat @ w[p + "uv"].t()).reshape(n, 3, 24)
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    mask = (j <= i) & (i - j < 9)
    out = []
    for head in range(3):
        scores = (q[:, head] @ k[:, head].t() * c["scale"]).masked_fill(~mask, -math.inf)
        scores = torch.cat([scores, w[p + "sink"][head].expand(n, 1)], 1)
        out.append(torch.softmax(scores, 1)[:, :n] @ v[:, head])
    want = torch.cat(out, 1) @ w[p + "o"].t()
    assert torch.allclose(torch.stack(got), want, rtol=1e-10, atol=1e-12)


def test_passes_keep_their_own_keys_and_memories():
    raw = copy.deepcopy(nu.SMALL_A)
    seq = pn.Model(raw, nu.make_weights(raw, seed=2)).start()
    seq.feed([1, 2, 3])
    assert [run for run, _ in sorted(seq.kept) if _ == "key"] == [1, 2, 3, 4, 5, 6, 8]
    assert {run for run, what in seq.state if what == "memory"} == {0, 7}
    assert all(len(after) == 9 for after in seq.stream_after)
    assert not torch.allclose(seq.kept[(1, "key")][0], seq.kept[(3, "key")][0])


# ---------------------------------------------------------------------------------------------------- configuration
def test_the_configuration_hands_on_every_size_and_constant():
    from cie_amd.cache.manager import FixedState, PagedKV
    from cie_amd.config import config_from_dict
    from cie_amd.parts.model import DecoderModel

    config = config_from_dict(copy.deepcopy(nu.SMALL_A))
    spec = config.model_spec()
    assert (spec.vocab_size, spec.hidden_size, len(spec.layers), spec.logit_scale) == (96, 64, 5, 1.5)
    assert [layer.block for layer in spec.layers] == ["sandwich_norm"] * 5 and all(l.norm1.kind == "layer_norm" for l in spec.layers)
    delta = spec.layers[0].mixer.as_dict()
    assert (delta["num_heads"], delta["num_kv_heads"], delta["head_dim"], delta["value_dim"], delta["taps"], delta["eps"]) == (4, 2, 12, 20, 3, 1e-3)
    latent = spec.layers[1].mixer.as_dict()
    assert (latent["num_heads"], latent["head_dim"], latent["rot_dim"], latent["value_dim"], latent["q_rank"], latent["kv_rank"],
            latent["scale"], latent["window"], latent["sink"]) == (3, 16, 8, 24, 40, 56, 0.3, 9, True)
    assert latent["position"].kind == "rotary_half" and latent["position"].as_dict()["scaling"] == (4.0, 64.0, 16.0, 1.0)
    attention = spec.layers[2].mixer.as_dict()
    assert (attention["num_heads"], attention["num_kv_heads"], attention["head_dim"], attention["value_dim"], attention["scale"],
            attention["differential"], attention["chunk"], attention["output_gate"]) == (4, 2, 16, 12, 0.35, 0.3, 11, True)
    assert attention["position"].as_dict()["rotary_dim"] == 8
    assert spec.layers[0].feed_forward.kind == "none" and spec.layers[1].feed_forward.as_dict()["intermediate_size"] == 72
    assert spec.layers[4].mixer.as_dict()["window"] is None
    # the run order: every run has a cache unit of its own, every pass begins with the joining step
    assert [(c.layer, c.cache, c.entry) for c in spec.order] == [(0, 0, None), (1, 1, 0), (2, 2, None), (1, 3, 1), (2, 4, None),
                                                                (1, 5, 2), (2, 6, None), (3, 7, None), (4, 8, None)]
    model = DecoderModel(spec)
    needs = model.cache_needs()
    assert needs[0] == (FixedState((4, 20, 12)), FixedState((4, 2, 44))) and needs[7] == (FixedState((3, 8, 20)), FixedState((3, 1, 48)))
    assert isinstance(needs[1], PagedKV) and needs[1].window == 9 and needs[1].kv_heads == 1 and needs[1] == needs[3] == needs[5]
    assert needs[2].window == 11 and needs[2].kv_heads == 2 and needs[8].window is None
    # a block's last kernel makes the first norm of what runs next, except in front of a pass
    assert [f is not None for f in model.followers] == [False, True, False, True, False, True, True, True, False]
    expected = model.expected_tensors()
    assert expected["loop.in"].shape == (64, 128) and expected["loop.step"].shape == (3, 64)
    assert expected["l0.mix.q.conv"].shape == (24, 3) and expected["l0.mix.v.conv"].shape == (80, 3) and expected["l0.mix.norm"].shape == (20,)
    assert expected["l1.mix.uq"].shape == (72, 40) and expected["l1.mix.dkv"].shape == (64, 64)
    assert expected["l2.mix.q"].shape == (128, 64) and expected["l2.mix.k"].shape == (64, 64) and expected["l2.mix.g"].shape == (48, 64)
    assert expected["l0.norm2"].optional and not expected["l1.norm2b.b"].optional
    assert config.to_hf_config()["architecture"] == "Nopunex"


def test_without_a_loop_there_is_no_joining_step_and_the_query_latent_may_be_the_checkpoints():
    from cie_amd.config import config_from_dict
    from cie_amd.parts.model import expected_tensors

    raw = nu.single(copy.deepcopy(nu.SMALL_A["layers"][1]))
    del raw["layers"][0]["mixer"]["q_rank"]
    expected = expected_tensors(config_from_dict(raw).model_spec())
    assert not any(name.startswith("loop") for name in expected)
    assert expected["l0.mix.dq"].shape == (None, 32) and expected["l0.mix.uq"].shape == (72, None)


@pytest.mark.parametrize("change, message", [
    (lambda r: r["layers"][0].update(type="delta_2"), "unknown layer type"),
    (lambda r: r["layers"][0]["mixer"].update(kv_heads=3), "no multiple"),
    (lambda r: r["layers"][0]["mixer"].update(conv=0), "positive integer"),
    (lambda r: r["layers"][0]["mixer"].update(dim=600), "512"),
    (lambda r: r["layers"][0]["mixer"].pop("vdim"), "missing"),
    (lambda r: r["layers"][1]["mixer"]["rot"].update(dims=16), "at most the head size"),
    (lambda r: r["layers"][1]["mixer"].update(kv_rank=2000), "latent"),
    (lambda r: r["layers"][1]["mixer"]["mask"].update(size=0), "positive integer"),
    (lambda r: r["layers"][2]["mixer"].pop("diff"), "missing"),
    (lambda r: r["layers"][2]["mixer"].update(heads=3), "no multiple"),
    (lambda r: r["layers"][1]["mlp"].update(kind="moe"), "unknown kind"),
    (lambda r: r["loop"].update(stop=6), "no run"),
    (lambda r: r["loop"].update(times=0), "positive integer"),
    (lambda r: r.pop("width"), "missing"),
])
def test_the_configuration_refuses_what_does_not_fit(change, message):
    from cie_amd.config import ConfigError, config_from_dict

    raw = copy.deepcopy(nu.SMALL_A)
    change(raw)
    with pytest.raises(ConfigError, match=message):
        config_from_dict(raw)


def test_random_weights_mode_draws_every_tensor():
    from cie_amd.config import config_from_dict
    from cie_amd.parts.model import expected_tensors
    from cie_amd.weights.loader import RandomSource

    for raw in nu.SMALL.values():
        expected = expected_tensors(config_from_dict(copy.deepcopy(raw)).model_spec())
        tensors = RandomSource(3).load(expected, "float32", "cpu")
        assert set(tensors) == {name for name, spec in expected.items() if not spec.optional}
        assert all(spec.fits(tuple(tensors[name].shape)) for name, spec in expected.items() if name in tensors)


def test_plans_of_the_delta_walk_hold_the_memory():
    from cie_amd.kernels import ops

    for dim, vdim in ((1, 1), (12, 20), (72, 24), (128, 128), (129, 200), (256, 256), (256, 700), (512, 33), (40, 1000)):
        rows, columns, threads, slice_cols, chunk = ops.plan_delta_walk(dim, vdim)
        assert 16 * rows >= dim and threads % 64 == 0 and 64 <= threads <= 512 and threads // 16 * columns >= slice_cols
        assert 1 <= chunk and 4 * chunk * (32 * rows + 2 * slice_cols + 3) <= 64 * 1024 and rows * columns <= ops.DELTA_STATE_NUMBERS
    with pytest.raises(ValueError):
        ops.plan_delta_walk(513, 8)
