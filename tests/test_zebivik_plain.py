"""The Zebivik design without a GPU: its configuration reader, the tensors it declares, what it asks of the cache, and the
plain implementation against itself and against its equations in another form (whole prompt against pieces through its
memory; both recurrences against their unrolled sums; the rotation, the slowed frequencies, the choice inside groups)."""
import copy
import math
import re

import pytest
import torch

import zebivik_configs as ZC
from plain import zebivik_plain as P

F64 = torch.float64


def random_weights(cfg, seed=0):
    from yalm_amd.config import config_from_dict
    from yalm_amd.engine.model import param_specs_of
    from yalm_amd.weights import random_init
    specs = param_specs_of(config_from_dict(cfg).to_spec())
    return {s.name: random_init.random_values(s.name, s.shape, s.init, s.fan_in, seed).to(F64) for s in specs}


def randn(*shape, seed=0):
    return torch.randn(*shape, dtype=F64, generator=torch.Generator().manual_seed(seed))


@pytest.mark.parametrize("name", sorted(ZC.ALL))
def test_configuration_round_trip(name):
    from yalm_amd.config import ZebivikConfig, config_from_dict
    cfg = config_from_dict(ZC.ALL[name])
    assert isinstance(cfg, ZebivikConfig)
    assert cfg.to_dict() == ZC.ALL[name]
    assert config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict()
    cfg.to_spec()


def test_parts_and_cache_lines():
    from yalm_amd.cache.manager import CacheManager, KVRequest, StateRequest
    from yalm_amd.config import config_from_dict
    from yalm_amd.engine.model import Model
    spec = config_from_dict(ZC.MIXED).to_spec()
    assert spec.layers[2].part("feed_forward") is None and spec.layers[2].part("feed_forward_out_norm") is None
    assert spec.layers[0].mixer_out_norm.params["result_scale"] == 0.7 and "result_scale" not in spec.final_norm.params
    assert spec.head.params["softcap"] == 20.0
    requests = Model(spec).cache_requests()
    assert requests[0] == {"left": KVRequest(2, 48), "right": StateRequest((3 * 12 * 20,))}
    assert requests[1] == {"conv": StateRequest((3, 120)), "state": StateRequest((120,))}
    assert requests[5] == {"left": KVRequest(1, 48), "right": StateRequest((7000,))}
    assert Model(config_from_dict(ZC.ODD).to_spec()).cache_requests()[0] == {"conv": None, "state": StateRequest((35,))}
    only = CacheManager(Model(config_from_dict(ZC.ONLY_LRU).to_spec()).cache_requests(), 64, 1000, torch.float32, "cpu", n_slots=2)
    assert only.unbounded and not only.kv_groups


def test_shared_products():
    """The two sides' first matrices stand one below the other, their last ones side by side; heads are spread to the cache's width,
    the gates' rows filled up to whole fours; a side's scale is not in the matrices."""
    from yalm_amd.config import config_from_dict
    from yalm_amd.engine.model import Model
    m = Model(config_from_dict(ZC.MIXED).to_spec())
    w = random_weights(ZC.MIXED)
    mixer = m.blocks[0].mixer
    rows = torch.cat([mixer.left.in_rows(w.get), mixer.right.in_rows(w.get)])
    assert rows.shape == (6 * 24 + 2 * 24 + 2 * 40 + 8 + 2 * 36 + 2 * 60, 80) == (mixer.left.n_in + mixer.right.n_in, 80)
    g = 6 * 24 + 2 * 24 + 2 * 40
    assert torch.equal(rows[g:g + 6], w["l0.mix.left.g"]) and float(rows[g + 6:g + 8].abs().max()) == 0.0
    assert torch.equal(rows[g + 8:g + 44], w["l0.mix.right.q"])
    cols = torch.cat([mixer.left.out_columns(w.get), mixer.right.out_columns(w.get)], dim=1)
    assert cols.shape == (80, 6 * 48 + 60)
    assert torch.equal(cols[:, :40], w["l0.mix.left.o"][:, :40]) and float(cols[:, 40:48].abs().max()) == 0.0
    assert torch.equal(cols[:, 288:], w["l0.mix.right.o"])


def test_declared_tensors():
    from yalm_amd.config import config_from_dict
    from yalm_amd.engine.model import param_specs_of
    shapes = {s.name: tuple(s.shape) for s in param_specs_of(config_from_dict(ZC.MIXED).to_spec())}
    assert shapes["embed"] == shapes["head"] == (211, 80)
    for n in ("embed.norm", "final.norm", "l0.norm1", "l0.norm1b", "l1.norm2", "l1.norm2b"):
        assert shapes[n] == shapes[n + ".b"] == (80,) and shapes[n + ".alpha"] == ()
    assert "l2.norm2" not in shapes and "l2.norm2b" not in shapes
    assert shapes["l0.mix.left.q"] == (144, 80) and shapes["l0.mix.left.k.b"] == (48,) and shapes["l0.mix.left.v"] == (80, 80)
    assert shapes["l0.mix.left.g"] == (6, 80) and shapes["l0.mix.left.o"] == (80, 240) and shapes["l0.mix.left.o.b"] == (80,)
    assert shapes["l0.mix.right.k"] == (36, 80) and shapes["l0.mix.right.g"] == (60, 80) and shapes["l0.mix.right.norm"] == (60,)
    assert "l0.mix.left.out" not in shapes and "l0.mix.right.q.b" not in shapes
    assert shapes["l1.mix.y"] == (120, 80) and shapes["l1.mix.conv"] == (120, 4) and shapes["l1.mix.ra"] == (5, 24, 24)
    assert shapes["l1.mix.ri.b"] == (5, 24) and shapes["l1.mix.lam"] == (120,) and shapes["l1.mix.o"] == (80, 120)
    assert shapes["l0.mlp.gate"] == (96, 80) and shapes["l1.mlp.correction"] == (15,) and shapes["l1.mlp.e14.down"] == (80, 48)
    assert shapes["l1.mlp.shared.up"] == (40, 80) and "l3.mlp.shared.up" not in shapes


@pytest.mark.parametrize("change,message", [
    (lambda c: c.pop("residual_mult"), "residual_mult"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c.update(logit_softcap=-1.0), "logit_softcap"),
    (lambda c: c["layers"][0].update(type="attention"), "not one of"),
    (lambda c: c["layers"][0]["mixer"].pop("left_scale"), "left_scale"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4), "multiple"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=26), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"]["scaling"].pop("high"), "high"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"]["scaling"].update(high=0.5), "high not below low"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5, 0.5]), "decay"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5, 0.5, 1.5]), "decay"),
    (lambda c: c["layers"][1]["mixer"].update(blocks=7), "multiple of blocks"),
    (lambda c: c["layers"][1]["mixer"].update(conv=0), "conv"),
    (lambda c: c["layers"][0]["mlp"].update(limit=0.0), "limit"),
    (lambda c: c["layers"][0]["mlp"].update(kind="mlp"), "neither"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=7), "do not go together"),
    (lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=4), "do not go together"),
    (lambda c: c["layers"][1]["mlp"]["shared"].update(ff=0), "do not go together"),
])
def test_configurations_that_are_refused(change, message):
    from yalm_amd.config import ConfigError, config_from_dict
    bad = copy.deepcopy(ZC.MIXED)
    change(bad)
    with pytest.raises(ConfigError) as e:
        config_from_dict(bad)
    assert re.search(message, str(e.value)), str(e.value)


def test_parts_that_do_not_go_together_are_refused():
    from yalm_amd.config import PartSpec
    from yalm_amd.parts import build_part
    attention = {"n_heads": 2, "n_kv_heads": 1, "key_dim": 8, "value_dim": 8}
    linear = PartSpec("lightning", {"n_heads": 1, "key_dim": 4, "decay": [0.5]})
    with pytest.raises(ValueError):                # an attention without a gate a head brings its result nowhere else
        build_part("mixer", PartSpec("side_by_side", {"left": PartSpec("shaped_attention", attention), "right": linear, "scales": (1.0, 1.0)}), 16, "")
    with pytest.raises(ValueError):
        build_part("mixer", PartSpec("lightning", {"n_heads": 2, "key_dim": 4, "decay": [0.5]}), 16, "")
    with pytest.raises(ValueError):
        build_part("mixer", PartSpec("rglru", {"width": 10, "blocks": 3, "taps": 2}), 16, "")
    with pytest.raises(ValueError):                # groups go with scores brought to one sum
        build_part("feed_forward", PartSpec("moe", {"hidden": 8, "n_experts": 4, "top": 2, "groups": 2, "up_shift": 0.0}), 16, "")
    with pytest.raises(ValueError):
        build_part("feed_forward", PartSpec("swiglu", {"hidden": 8, "alpha": 1.7}), 16, "")
    biased = build_part("mixer", PartSpec("shaped_attention", dict(attention, out_bias=True)), 16, "")
    biased.late_bias = torch.zeros(16)
    with pytest.raises(ValueError):                # nobody would add the bias
        biased.forward(None, None, None, 0)
    with pytest.raises(ValueError):
        biased.forward_to(None, None, None, 0)


@pytest.mark.parametrize("name", sorted(ZC.ALL))
@pytest.mark.parametrize("pieces", [[40], [1] * 40, [2] * 20, [7, 1, 30, 2], [39, 1]])
def test_plain_whole_text_equals_its_pieces(name, pieces):
    cfg = ZC.ALL[name]
    w = random_weights(cfg, seed=2)
    tokens = torch.randint(0, cfg["vocab"], (40,), generator=torch.Generator().manual_seed(1)).tolist()
    whole = P.forward(cfg, w, tokens)
    memory, rows, at = {}, [], 0
    for n in pieces:
        rows.append(P.forward(cfg, w, tokens[at:at + n], memory=memory, start=at))
        at += n
    assert torch.allclose(torch.cat(rows), whole, rtol=1e-9, atol=1e-9)


def test_plain_linear_attention_is_its_unrolled_sum():
    T, d, dv, g = 9, 4, 3, 0.8
    q, k, v = randn(T, d), randn(T, d, seed=1), randn(T, dv, seed=2)
    out, S = P.decay_scan(q, k, v, g, torch.zeros(d, dv, dtype=F64))
    for t in range(T):
        assert torch.allclose(out[t], sum(g ** (t - s) * (q[t] @ k[s]) * v[s] for s in range(t + 1)))
    assert torch.allclose(S, sum(g ** (T - 1 - s) * torch.outer(k[s], v[s]) for s in range(T)))


def test_plain_gated_recurrence_is_its_unrolled_sum():
    T, C = 7, 5
    u, r, i, lam = randn(T, C), torch.sigmoid(randn(T, C, seed=1)), torch.sigmoid(randn(T, C, seed=2)), randn(C, seed=3)
    out, S = P.lru_scan(u, r, i, lam, torch.zeros(C, dtype=F64))
    a = torch.exp(-8.0 * r * torch.nn.functional.softplus(lam))
    for t in range(T):
        want = sum(a[s + 1:t + 1].prod(dim=0) * torch.sqrt(1 - a[s] ** 2) * i[s] * u[s] for s in range(t + 1))
        assert torch.allclose(out[t], want)
    assert torch.equal(S, out[-1])


def test_plain_convolution_and_block_gates():
    x, w, b = randn(6, 3), randn(3, 4, seed=1), randn(3, seed=2)
    out = P.causal_conv(x, w, b, {})
    for t in range(6):
        want = b + sum(w[:, 3 - j] * x[t - j] for j in range(4) if t - j >= 0)
        assert torch.allclose(out[t], want)
    u, m, mb = randn(2, 6), randn(2, 3, 3, seed=3), randn(2, 3, seed=4)
    z = torch.cat([u[:, :3] @ m[0].T + mb[0], u[:, 3:] @ m[1].T + mb[1]], dim=1)
    assert torch.allclose(P.block_gate(u, m, mb), torch.sigmoid(z))


def test_plain_rotation_turns_halves_and_slows_long_wavelengths():
    x = torch.zeros(1, 1, 7, dtype=F64)
    x[0, 0, 1], x[0, 0, 6] = 1.0, 2.0              # element 1 goes with element 3 of four
    rot = {"dims": 4, "base": 100.0}
    y = P.rotate(x, torch.tensor([3]), rot)[0, 0]
    a = 3 * 100.0 ** -0.5
    assert torch.allclose(y, torch.tensor([0, math.cos(a), 0, math.sin(a), 0, 0, 2.0], dtype=F64))
    rot = {"dims": 64, "base": 10000.0}
    plain, slow = P.frequencies(rot), P.frequencies(dict(rot, scaling={"factor": 8.0, "low": 1.0, "high": 4.0, "original": 256}))
    wave = 2 * math.pi / plain
    for f, s, l in zip(plain.tolist(), slow.tolist(), wave.tolist()):
        if l < 64:
            assert s == f
        elif l > 256:
            assert abs(s - f / 8) < 1e-15
        else:
            mix = (256 / l - 1.0) / 3.0
            assert abs(s - ((1 - mix) * f / 8 + mix * f)) < 1e-15
    assert (wave < 64).any() and (wave > 256).any() and ((wave > 64) & (wave < 256)).any()


def test_plain_frequencies_match_the_library():
    from yalm_amd.parts.rope import inverse_frequencies
    for dims, base, sc in ((32, 500.0, (4.0, 1.0, 4.0, 64)), (64, 5000.0, (3.0, 2.0, 2.0, 100)), (10, 1e6, None)):
        rot = {"dims": dims, "base": base}
        lib = None
        if sc:
            rot["scaling"] = dict(zip(("factor", "low", "high", "original"), sc))
            lib = {"rope_type": "llama3", "factor": sc[0], "low_freq_factor": sc[1], "high_freq_factor": sc[2], "original_max_position_embeddings": sc[3]}
        assert torch.allclose(P.frequencies(rot), inverse_frequencies(dims, dims, base, lib), rtol=1e-12)


def test_plain_norm_has_no_mean():
    w = {"n": torch.tensor([2.0, 3.0]), "n.b": torch.tensor([0.5, -1.0]), "n.alpha": torch.tensor(0.3)}
    y = P.norm(torch.tensor([[1.0, 100.0]], dtype=F64), w, "n")
    assert torch.allclose(y, torch.tensor([[math.tanh(0.3) * 2 + 0.5, 2.0]], dtype=F64))


def test_plain_clamped_unit():
    w = {"gate": torch.tensor([[1.0], [1.0]]), "up": torch.tensor([[1.0], [-1.0]]), "down": torch.eye(2)}
    y = P.clamped_unit(torch.tensor([[5.0], [-5.0]], dtype=F64), 2.0, w, "")
    unit = lambda g, u: g / (1 + math.exp(-1.702 * g)) * (u + 1)
    assert torch.allclose(y, torch.tensor([[unit(2, 2), unit(2, -2)], [unit(-5, -2), unit(-5, 2)]], dtype=F64))


def test_plain_choice_inside_groups():
    """Four groups of two; a group counts by its largest choice score; corrections make the choice and not the weights; a
    group outside the kept ones gives nothing, also where every choice score is negative."""
    z = torch.tensor([[2.0, -3.0, 0.5, 0.4, -1.0, -1.0, 1.9, 0.0]], dtype=F64)
    w = {"router": torch.eye(8, dtype=F64), "correction": torch.tensor([-2.0, -2.0, -1.0, -1.0, -3.0, -3.0, -1.5, -1.2], dtype=F64)}
    router = {"experts": 8, "top": 3, "scale": 2.0, "groups": {"count": 4, "keep": 2}}
    s = torch.softmax(z, -1)[0]
    c = s + w["correction"]
    groups = sorted(range(4), key=lambda g: -float(max(c[2 * g], c[2 * g + 1])))[:2]
    want = sorted([e for e in range(8) if e // 2 in groups], key=lambda e: -float(c[e]))[:3]
    chosen, weight = P.route(z, router, w, "")
    assert chosen[0].tolist() == want and float(c.max()) < 0
    assert torch.allclose(weight[0], s[want] / s[want].sum() * 2.0) and abs(float(weight.sum()) - 2.0) < 1e-12


def test_the_measured_configurations_are_valid():
    """bench.py --design zebivik builds these."""
    import os
    import sys
    sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
    import bench
    from yalm_amd.config import config_from_dict
    for width in (2048, 4096):
        cfg = config_from_dict(bench.zebivik_config(width))
        cfg.to_spec()
        assert {l["type"] for l in cfg.layers} == {"parallel", "rglru"}
        assert {l["mlp"]["kind"] for l in cfg.layers} == {"dense", "moe"}
