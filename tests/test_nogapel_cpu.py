"""CPU: what pins the plain Nogapel implementation (tests/plain_nogapel.py), and the configuration's reading, which needs no
GPU."""

from __future__ import annotations

import copy
import math

import pytest
import torch

import nogapel_util as gu
import plain_nogapel as pg

F = torch.float64


def test_norms_and_activations_against_the_library():
    x, w = torch.randn(5, 12, dtype=F) * 3, torch.rand(12, dtype=F) + 0.5
    assert torch.allclose(pg.rms_norm(x, w, 1e-3), torch.nn.functional.rms_norm(x, (12,), w, 1e-3), rtol=1e-12)
    assert torch.allclose(pg.gelu_tanh(x), torch.nn.functional.gelu(x, approximate="tanh"), rtol=1e-12, atol=1e-14)
    assert torch.equal(pg.squared_relu(x), torch.relu(x) ** 2)


@pytest.mark.parametrize("taps", [1, 2, 5])
def test_the_short_convolution_is_the_librarys(taps):
    u, w = torch.randn(4, 3, dtype=F), torch.randn(3, taps, dtype=F)
    padded = torch.cat([torch.zeros(taps - 1, 3, dtype=F), u]).t()[None]
    want = torch.nn.functional.conv1d(padded, w[:, None, :], groups=3)[0].t()
    assert torch.allclose(pg.short_convolution(u, w), want, rtol=1e-12, atol=1e-14)


def test_rotation_of_neighbours_is_a_complex_multiplication():
    heads = torch.randn(9, 3, 10, dtype=F)
    rates = pg.frequencies({"dims": 6, "base": 100.0})
    assert torch.allclose(rates, 100.0 ** (-torch.arange(3, dtype=F) * 2 / 6))
    turned = pg.rotate(heads, rates)
    z = torch.complex(heads[..., 0:6:2], heads[..., 1:6:2])
    z = z * torch.polar(torch.ones(9, 1, 3, dtype=F), torch.arange(9, dtype=F)[:, None, None] * rates)
    assert torch.allclose(turned[..., 0:6:2], z.real, atol=1e-13) and torch.allclose(turned[..., 1:6:2], z.imag, atol=1e-13)
    assert torch.equal(turned[..., 6:], heads[..., 6:])


def test_frequencies_divided_by_wavelength_against_the_package():
    """Short waves stay, long ones are divided, those between are a weighted mean; the part's float32 rates are the same."""
    from cie_amd.parts.position import RotaryPairs

    for rot in ({"dims": 24, "base": 1000.0, "scaling": gu.BANDS},
                {"dims": 64, "base": 1e4, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 2048}}):
        plain, rates = pg.frequencies({k: rot[k] for k in ("dims", "base")}), pg.frequencies(rot)
        s = rot["scaling"]
        wavelength = 2 * math.pi / plain
        short, long = wavelength < s["original"] / s["high"], wavelength > s["original"] / s["low"]
        between = ~short & ~long
        assert short.any() and long.any() and between.any()
        assert torch.equal(rates[short], plain[short]) and torch.allclose(rates[long], plain[long] / s["factor"], rtol=1e-13)
        assert bool((rates[between] < plain[between]).all()) and bool((rates[between] > plain[between] / s["factor"]).all())
        got, gain = RotaryPairs(rot["dims"], rot["base"], None, bands=(s["factor"], s["low"], s["high"], s["original"])).inv_freq()
        assert gain == 1.0 and torch.allclose(got.double(), rates, rtol=1e-6)
    # exactly between the bounds: a wave that turns (low + high) / 2 times over the original length
    base = (2 * math.pi * 2.5 / 100) ** -2.0  # pair 1 of 4 dims: rate base^(-1/2) = 2 pi 2.5 / 100
    mid = pg.frequencies({"dims": 4, "base": base, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 100}})[1]
    assert abs(float(mid) / (2 * math.pi * 2.5 / 100) - (0.5 + 0.5 / 4)) < 1e-12


def test_rotation_tables_with_and_without_bands_do_not_meet():
    from cie_amd.parts.position import RotaryPairs

    bands = (5.0, 0.5, 3.0, 64.0)
    plain, banded = RotaryPairs(16, 1000.0, None), RotaryPairs(16, 1000.0, None, bands=bands)
    cos, _ = plain.tables(torch.device("cpu"), 10)
    other, _ = banded.tables(torch.device("cpu"), 10)
    assert not torch.equal(cos, other) and torch.equal(other, (torch.arange(other.shape[0], dtype=torch.float32)[:, None] * banded.inv_freq()[0]).cos())
    with pytest.raises(ValueError, match="bands"):
        RotaryPairs(16, 1000.0, None, bands=(4.0, 4.0, 1.0, 64.0))


def test_masks_and_the_sink():
    m = pg.mask(6, 3)
    assert m[4].tolist() == [False, False, True, True, True, False] and pg.mask(6)[5].all() and not pg.mask(6)[4, 5]
    assert pg.mask(4, 1).equal(torch.eye(4, dtype=torch.bool))
    scores, sink = torch.randn(6, 6, dtype=F), torch.tensor(0.7, dtype=F)
    full = torch.cat([scores.masked_fill(~m, -math.inf), sink.expand(6, 1)], 1)
    assert torch.allclose(pg.softmax(scores, m, sink), torch.softmax(full, 1)[:, :6], rtol=1e-13)


def test_attention_against_library_attention():
    """One layer's mixer, composed from library calls."""
    raw = gu.single(copy.deepcopy(gu.SMALL_A["layers"][1]), width=40)
    w = {k: v.double() for k, v in gu.make_weights(raw, seed=2).items()}
    c, p, n = raw["layers"][0]["mixer"], "l0.mix.", 20
    h = torch.randn(n, 40, dtype=F)
    first = torch.randn(n, 24, dtype=F)
    for carried, mixed in (({}, False), ({"first": first}, True)):
        share = torch.tensor(0.3, dtype=F)
        got = pg.attention({**w, p + "vmix": share}, p, c, h, 1e-6, carried)
        conv = lambda name: torch.nn.functional.conv1d(torch.cat([torch.zeros(2, w[p + name].shape[0], dtype=F), h @ w[p + name].t()]).t()[None],
                                                       w[f"{p}{name}.conv"][:, None], groups=w[p + name].shape[0])[0].t()
        norm = lambda x, name: torch.nn.functional.rms_norm(x, (24,), w[p + name], 1e-6)
        rates = pg.frequencies(c["rot"])
        q = pg.rotate(norm(conv("q").reshape(n, 4, 24), "q.norm"), rates).transpose(0, 1)
        k = pg.rotate(norm(conv("k").reshape(n, 2, 24), "k.norm"), rates).transpose(0, 1).repeat_interleave(2, 0)
        v = conv("v")
        if mixed:
            v = 0.7 * v + 0.3 * first
        else:
            assert torch.equal(carried["first"], v) or torch.allclose(carried["first"], v, rtol=1e-12, atol=1e-13)
        v = v.reshape(n, 2, 12).transpose(0, 1).repeat_interleave(2, 0)
        want = torch.nn.functional.scaled_dot_product_attention(q, k, v, attn_mask=pg.mask(n, 9), scale=c["scale"])
        assert torch.allclose(got, want.transpose(0, 1).reshape(n, 48) @ w[p + "o"].t(), rtol=1e-9, atol=1e-11)


def test_latent_attention_against_library_attention_on_expanded_keys():
    raw = gu.single(copy.deepcopy(gu.SMALL_A["layers"][2]), width=64)
    w = {k: v.double() for k, v in gu.make_weights(raw, seed=2).items()}
    c, p, n = raw["layers"][0]["mixer"], "l0.mix.", 20
    h = torch.randn(n, 64, dtype=F)
    got = pg.latent_attention(w, p, c, h, 1e-6, {})
    rates = pg.frequencies(c["rot"])
    rms = lambda x, g: torch.nn.functional.rms_norm(x, (x.shape[-1],), g, 1e-6)
    q = (rms(h @ w[p + "dq"].t(), w[p + "dq.norm"]) @ w[p + "uq"].t()).reshape(n, 3, 24)
    q = torch.cat([q[..., :16], pg.rotate(q[..., 16:], rates)], -1)
    down = h @ w[p + "dkv"].t()
    lat = rms(down[:, :56], w[p + "dkv.norm"])
    k = torch.cat([(lat @ w[p + "uk"].t()).reshape(n, 3, 16), pg.rotate(down[:, 56:], rates)[:, None].expand(n, 3, 8)], -1)
    v = (lat @ w[p + "uv"].t()).reshape(n, 3, 24)
    # the sink as one more key whose score is the sink and whose value is zero
    out = []
    for i in range(3):
        scores = (q[:, i] @ k[:, i].t() * c["scale"]).masked_fill(~pg.mask(n), -math.inf)
        scores = torch.cat([scores, w[p + "sink"][i].expand(n, 1)], 1)
        out.append(torch.softmax(scores, 1)[:, :n] @ v[:, i])
    assert torch.allclose(got, torch.cat(out, 1) @ w[p + "o"].t(), rtol=1e-10, atol=1e-12)


def test_a_model_composed_by_hand():
    """The first token of a model of two attention layers (every softmax is one, a convolution has its last tap alone): the
    norm on the embedding, one norm for both sublayers, the token's own branch behind them, the values of the first layer in
    the second."""
    layers = [copy.deepcopy(gu.SMALL_A["layers"][1]), copy.deepcopy(gu.SMALL_A["layers"][1])]
    raw = gu.single(*layers, width=40)
    w = {k: v.double() for k, v in gu.make_weights(raw, seed=1).items()}
    rms = lambda x, name: x / torch.sqrt((x * x).mean() + 1e-6) * w[name]
    x = rms(w["embed"][3], "embed.norm")
    first = None
    for i in range(2):
        p = f"l{i}."
        h = rms(x, p + "norm1")
        v = (w[p + "mix.v"] @ h) * w[p + "mix.v.conv"][:, -1]
        first = v if first is None else first
        share = w[p + "mix.vmix"] if i else 0.0
        v = ((1 - share) * v + share * first).reshape(2, 12).repeat_interleave(2, 0).reshape(-1)
        x = x + w[p + "mix.o"] @ v + w[p + "mlp.down"] @ (torch.relu(w[p + "mlp.up"] @ h) ** 2)
        y = w[p + "side.proj"] @ (torch.nn.functional.gelu(w[p + "side.gate"] @ x, approximate="tanh") * w["side.embed"][3, 8 * i: 8 * i + 8])
        x = x + rms(y, p + "side.norm")
    assert torch.allclose(pg.forward(raw, w, [3])[0], w["head"] @ rms(x, "final.norm"), rtol=1e-10, atol=1e-12)


def test_a_prefix_does_not_know_what_follows():
    raw = gu.SMALL_A
    w = gu.make_weights(raw, seed=4)
    tokens = [int(t) for t in torch.randint(0, 96, (40,), generator=torch.Generator().manual_seed(1))]
    whole = pg.forward(raw, w, tokens)
    for n in (1, 2, 9, 39):
        assert torch.allclose(pg.forward(raw, w, tokens[:n]), whole[:n], rtol=1e-9, atol=1e-11)


# ---------------------------------------------------------------------------------------------------- configuration
def test_the_configuration_hands_on_every_size_and_constant():
    from cie_amd.cache.manager import FixedState, PagedKV
    from cie_amd.config import config_from_dict
    from cie_amd.parts.model import DecoderModel

    config = config_from_dict(copy.deepcopy(gu.SMALL_A))
    spec = config.model_spec()
    assert (spec.vocab_size, spec.hidden_size, len(spec.layers), spec.side_table_columns) == (96, 64, 6, 72)
    assert all(layer.block == "parallel" and layer.norm1.as_dict() == {"size": 64, "eps": 1e-3} for layer in spec.layers)
    assert spec.embedding_norm == spec.final_norm == spec.layers[0].norm1
    assert [layer.side.as_dict()["index"] for layer in spec.layers] == list(range(6)) and spec.layers[0].side.as_dict()["dim"] == 12
    mixers = [layer.mixer.as_dict() for layer in spec.layers]
    first = mixers[1]
    assert (first["num_heads"], first["num_kv_heads"], first["head_dim"], first["value_dim"], first["scale"], first["window"],
            first["conv_taps"], first["qk_norm"], first["eps"]) == (4, 2, 24, 12, 0.25, 9, 3, "weight", 1e-3)
    rotation = first["position"]
    assert rotation.kind == "rotary_pairs" and rotation.as_dict()["bands"] == (5.0, 0.5, 3.0, 64.0)
    assert rotation.as_dict()["rotary_dim"] == 24 and rotation.as_dict()["theta"] == 1000.0
    assert mixers[0]["position"].as_dict()["bands"] is None and mixers[0]["position"].as_dict()["rotary_dim"] == 10
    assert [m.get("value_mix") for m in mixers] == [None, "first", None, "mixed", None, "mixed"]
    latent = mixers[2]
    assert (latent["num_heads"], latent["head_dim"], latent["rot_dim"], latent["value_dim"], latent["q_rank"], latent["kv_rank"],
            latent["scale"], latent["window"], latent["sink"]) == (3, 16, 8, 24, 40, 56, 0.3, None, True)
    assert latent["position"].kind == "rotary_pairs" and latent["position"].as_dict()["bands"] == (5.0, 0.5, 3.0, 64.0)
    assert [layer.feed_forward.kind for layer in spec.layers] == ["dense_mlp"] * 3 + ["none"] + ["dense_mlp"] * 2
    assert spec.layers[1].feed_forward.as_dict()["intermediate_size"] == 72
    assert [(c.layer, c.cache, c.writes) for c in spec.order] == [(i, i, True) for i in range(6)]
    model = DecoderModel(spec)
    needs = model.cache_needs()
    assert isinstance(needs[1], tuple) and needs[1][0].window == 9 and needs[1][1] == FixedState((2, 4 * 24 + 2 * 24 + 2 * 12))
    assert needs[0][1] == FixedState((1, 6 * 16 + 3 * 16 + 3 * 20)) and isinstance(needs[2], PagedKV) and needs[2].window is None
    expected = model.expected_tensors()
    assert expected["side.embed"].shape == (96, 72) and expected["embed.norm"].shape == (64,)
    assert expected["l1.mix.q.conv"].shape == (96, 3) and expected["l1.mix.v.conv"].shape == (24, 3) and expected["l1.mix.k.norm"].shape == (24,)
    assert expected["l1.mix.vmix"].shape == () and expected["l1.mix.vmix"].optional and not expected["l3.mix.vmix"].optional
    assert "l0.mix.vmix" not in expected and "l3.mlp.up" not in expected and "l0.norm2" not in expected
    assert expected["l2.mix.uq"].shape == (72, 40) and expected["l2.side.gate"].shape == (12, 64) and expected["l2.side.proj"].shape == (64, 12)
    assert [block.joined for block in model.blocks] == [True, True, True, False, True, True]
    assert config.to_hf_config()["architecture"] == "Nogapel"


def test_parts_that_a_file_leaves_out():
    """No token table, no convolution, no rotation, one key head for every query head, a query latent of the checkpoint's."""
    from cie_amd.config import config_from_dict
    from cie_amd.parts.model import expected_tensors

    plain = {"type": "attention", "mixer": {"heads": 3, "dim": 8, "vdim": 8, "scale": 0.4}}
    expected = expected_tensors(config_from_dict(gu.single(plain, side=None)).model_spec())
    assert not any("side" in name or "conv" in name or "vmix" in name for name in expected) and expected["l0.mix.k"].shape == (24, 32)
    latent = copy.deepcopy(gu.SMALL_A["layers"][2])
    del latent["mixer"]["q_rank"]
    expected = expected_tensors(config_from_dict(gu.single(latent)).model_spec())
    assert expected["l0.mix.dq"].shape == (None, 32) and expected["l0.mix.uq"].shape == (72, None)


@pytest.mark.parametrize("change, message", [
    (lambda r: r["layers"][0].update(type="attention_2"), "unknown layer type"),
    (lambda r: r["layers"][0]["mixer"].update(kv_heads=4), "no multiple"),
    (lambda r: r["layers"][0]["mixer"].update(conv=0), "positive integer"),
    (lambda r: r["layers"][0]["mixer"].update(conv=17), "taps"),
    (lambda r: r["layers"][0]["mixer"].update(dim=300), "up to 256"),
    (lambda r: r["layers"][0]["mixer"].pop("vdim"), "missing"),
    (lambda r: r["layers"][1]["mixer"]["rot"].update(dims=26), "at most the head size"),
    (lambda r: r["layers"][1]["mixer"]["rot"]["scaling"].pop("low"), "missing"),
    (lambda r: r["layers"][1]["mixer"]["rot"]["scaling"].update(low=3.0), "low < high"),
    (lambda r: r["layers"][1]["mixer"]["mask"].update(size=0), "positive integer"),
    (lambda r: r["layers"][2]["mixer"].update(kv_rank=2000), "latent"),
    (lambda r: r["layers"][3]["mixer"].update(vdim=23), "cannot be mixed"),
    (lambda r: r["layers"][1]["mlp"].update(kind="moe"), "unknown kind"),
    (lambda r: r["token_side"].update(dim=0), "positive integer"),
    (lambda r: r.pop("width"), "missing"),
])
def test_the_configuration_refuses_what_does_not_fit(change, message):
    from cie_amd.config import ConfigError, config_from_dict

    raw = copy.deepcopy(gu.SMALL_A)
    change(raw)
    with pytest.raises(ConfigError, match=message):
        config_from_dict(raw)


def test_random_weights_mode_draws_every_tensor():
    from cie_amd.config import config_from_dict
    from cie_amd.parts.model import expected_tensors
    from cie_amd.weights.loader import RandomSource

    for raw in gu.SMALL.values():
        expected = expected_tensors(config_from_dict(copy.deepcopy(raw)).model_spec())
        tensors = RandomSource(3).load(expected, "float32", "cpu")
        assert set(tensors) == {name for name, spec in expected.items() if not spec.optional}
        assert all(spec.fits(tuple(tensors[name].shape)) for name, spec in expected.items() if name in tensors)


def test_joined_products_hold_both_parts_weights():
    """A block whose mixer and feed-forward share two products: the parts' own weights are gone, the shared ones hold them at
    places that start at multiples of 16 bytes."""
    from cie_amd.config import config_from_dict
    from cie_amd.parts.model import DecoderModel

    raw = gu.single(copy.deepcopy(gu.SMALL_A["layers"][5]), copy.deepcopy(gu.SMALL_A["layers"][4]), width=32)
    weights = gu.make_weights(raw, seed=2)
    model = DecoderModel(config_from_dict(raw).model_spec()).load(gu.Fixed(weights), "float32", "cpu")
    for index, (block, names) in enumerate(zip(model.blocks, (("q", "k", "v"), ("dq", "dkv")))):
        p = f"l{index}."
        up = weights[p + "mlp.up"]
        assert block.joined and block.inner % 8 == 0 and block.inner >= up.shape[0] and block.mixer.w_in is None and block.feed_forward.w_up is None
        assert (block.w_in.shape[0] - block.inner) % 8 == 0
        assert torch.equal(block.w_in[-block.inner:][: up.shape[0]], up) and float(block.w_in[-block.inner:][up.shape[0]:].abs().sum()) == 0.0
        first = weights[f"{p}mix.{names[0]}"]
        assert torch.equal(block.w_in[: first.shape[0]], first)
        down = weights[p + "mlp.down"]
        assert torch.equal(block.w_out[:, : down.shape[1]], down) and float(block.w_out[:, down.shape[1]: block.inner].abs().sum()) == 0.0
