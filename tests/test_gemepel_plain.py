"""The Gemepel design without a GPU: its configuration reader, the tensors it declares, what it asks of the cache, and the
plain implementation against itself and against its equations in another form (whole prompt against pieces through its
memory; the recurrence against its unrolled sum; the attention in the latent space; the choice inside groups)."""
import copy
import re

import pytest
import torch

import gemepel_configs as GC
from plain import gemepel_plain as P

F64 = torch.float64


def random_weights(cfg, seed=0):
    from yalm_amd.config import config_from_dict
    from yalm_amd.engine.model import param_specs_of
    from yalm_amd.weights import random_init
    specs = param_specs_of(config_from_dict(cfg).to_spec())
    return {s.name: random_init.random_values(s.name, s.shape, s.init, s.fan_in, seed).to(F64) for s in specs}


def randn(*shape, seed=0):
    return torch.randn(*shape, dtype=F64, generator=torch.Generator().manual_seed(seed))


@pytest.mark.parametrize("name", sorted(GC.ALL))
def test_configuration_round_trip(name):
    from yalm_amd.config import GemepelConfig, config_from_dict
    cfg = config_from_dict(GC.ALL[name])
    assert isinstance(cfg, GemepelConfig)
    assert config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict()
    cfg.to_spec()


def test_schedule_parts_and_cache_lines():
    from yalm_amd.cache.manager import KVRequest, StateRequest
    from yalm_amd.config import config_from_dict
    from yalm_amd.engine.model import Model
    spec = config_from_dict(GC.MIXED).to_spec()
    assert [(e.layer, e.cache, e.writes_cache) for e in spec.schedule] == \
        [(0, 0, True), (1, 1, True), (2, 0, False), (3, 3, True), (4, 4, True), (5, 0, False), (6, 6, True)]
    assert spec.layers[2].part("feed_forward") is None and spec.layers[2].part("feed_forward_norm") is None
    assert spec.layers[0].mixer_norm.params["stream_scale"] == 1.7 and "stream_scale" not in spec.final_norm.params
    requests = Model(spec).cache_requests()
    assert requests["embedding"].dtype == torch.int32
    assert requests[0] == KVRequest(1, 48) and requests[4] == KVRequest(1, 32) and 2 not in requests and 5 not in requests
    assert requests[1] == StateRequest((5 * 12 * 20,)) and requests[6] == StateRequest((7000,))
    assert "embedding" not in Model(config_from_dict(GC.ONLY_GLA).to_spec()).cache_requests()


def test_declared_tensors():
    from yalm_amd.config import config_from_dict
    from yalm_amd.engine.model import param_specs_of
    shapes = {s.name: tuple(s.shape) for s in param_specs_of(config_from_dict(GC.MIXED).to_spec())}
    assert shapes["embed"] == (211, 80) and shapes["bigram"] == (38, 80) and shapes["head"] == (211, 80)
    assert shapes["final.norm"] == shapes["final.norm.b"] == shapes["l6.norm2.b"] == (80,)
    assert shapes["l0.mix.dq"] == (20, 80) and shapes["l0.mix.dq.norm"] == (20,) and shapes["l0.mix.uq"] == (72, 20)
    assert shapes["l0.mix.dkv"] == (48, 80) and shapes["l0.mix.dkv.norm"] == (40,) and shapes["l0.mix.o"] == (80, 72)
    assert "l2.mix.dkv" not in shapes and "l2.mix.dkv.norm" not in shapes and shapes["l2.mix.uk"] == (40, 40)
    assert shapes["l1.mix.a1"] == (7, 80) and shapes["l1.mix.a2"] == (60, 7) and shapes["l1.mix.a2.b"] == (60,)
    assert shapes["l1.mix.g"] == (100, 80) and shapes["l1.mix.norm"] == (20,)
    assert shapes["l0.mlp.router"] == (12, 80) and shapes["l0.mlp.correction"] == (12,) and shapes["l0.mlp.e11.down"] == (80, 48)
    assert "l0.mlp.e0.gate" not in shapes and "l2.norm2" not in shapes and "l2.norm1.b" in shapes


def test_the_rank_of_the_decays_comes_from_the_tensors(tmp_path):
    """A folder's config.json need not name decay_rank: the rows of `a1` give it."""
    import json
    import os
    from yalm_amd.config import ConfigError, config_from_dict, config_from_folder
    from yalm_amd.weights import write_random_model
    folder = write_random_model(str(tmp_path / "m"), GC.MIXED, seed=1)
    f = os.path.join(folder, "config.json")
    with open(f) as fh:
        d = json.load(fh)
    for l in d["layers"]:
        l["mixer"].pop("decay_rank", None)
    with open(f, "w") as fh:
        json.dump(d, fh)
    cfg = config_from_folder(folder)
    assert [l["mixer"]["decay_rank"] for l in cfg.layers if l["type"] == "gla"] == [7, 16, 40]
    assert cfg.to_dict() == config_from_dict(GC.MIXED).to_dict()
    with pytest.raises(ConfigError):
        config_from_dict(d).to_spec()


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][2]["mixer"].update(kv_from=2), "earlier"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "earlier latent"),
    (lambda c: c["layers"][5]["mixer"].update(kv_from=2), "makes its own"),
    (lambda c: c["layers"][2]["mixer"].update(kv_rank=24), "differs"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(base=77.0), "differs"),
    (lambda c: c["layers"][0]["mixer"].update(rot_dim=7), "even"),
    (lambda c: c["layers"][0]["mixer"].pop("q_rank"), "q_rank"),
    (lambda c: c["layers"][1]["mixer"].update(tau=0.0), "tau"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=7), "do not go together"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=5), "do not go together"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=5), "do not go together"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "moe"),
    (lambda c: c["layers"][0].update(type="attention"), "not one of"),
    (lambda c: c.pop("postln_alpha"), "postln_alpha"),
    (lambda c: c["embedding"]["bigram"].update(buckets=0), "buckets"),
    (lambda c: c["embedding"]["bigram"].pop("mul_cur"), "mul_cur"),
])
def test_configurations_that_are_refused(change, message):
    from yalm_amd.config import ConfigError, config_from_dict
    bad = copy.deepcopy(GC.MIXED)
    change(bad)
    with pytest.raises(ConfigError) as e:
        config_from_dict(bad)
    assert re.search(message, str(e.value)), str(e.value)


@pytest.mark.parametrize("name", sorted(GC.ALL))
@pytest.mark.parametrize("pieces", [[40], [1] * 40, [2] * 20, [7, 1, 30, 2], [39, 1]])
def test_plain_whole_text_equals_its_pieces(name, pieces):
    cfg = GC.ALL[name]
    w = random_weights(cfg, seed=2)
    tokens = torch.randint(0, cfg["vocab"], (40,), generator=torch.Generator().manual_seed(1)).tolist()
    whole = P.forward(cfg, w, tokens)
    memory, rows, at = {}, [], 0
    for n in pieces:
        rows.append(P.forward(cfg, w, tokens[at:at + n], memory=memory, start=at))
        at += n
    assert torch.allclose(torch.cat(rows), whole, rtol=1e-9, atol=1e-9)


def test_plain_layer_norm_and_the_weighted_sum():
    x = randn(3, 11) * 4 + 2
    n = P.layer_norm(x, torch.ones(11, dtype=F64), torch.zeros(11, dtype=F64), 0.0)
    assert torch.allclose(n.mean(-1), torch.zeros(3, dtype=F64), atol=1e-12)
    assert torch.allclose((n * n).mean(-1), torch.ones(3, dtype=F64))
    assert torch.allclose(P.layer_norm(x, randn(11, seed=1), randn(11, seed=2), 1e-5),
                          torch.nn.functional.layer_norm(x, (11,), randn(11, seed=1), randn(11, seed=2), 1e-5), rtol=1e-12, atol=1e-12)


def test_plain_pairs():
    bigram = {"buckets": 10, "mul_prev": 7, "mul_cur": 3}
    assert P.pair_row(None, 4, bigram) == 10
    assert P.pair_row(2, 4, bigram) == (14 + 12) % 10
    w = {"embed": randn(20, 5), "bigram": randn(11, 5, seed=1)}
    memory = {}
    x = P.embed([4, 2, 2], {"scale": 0.5, "bigram": bigram}, w, memory)
    assert torch.allclose(x[0], w["embed"][4] * 0.5 + w["bigram"][10])
    assert torch.allclose(x[1], w["embed"][2] * 0.5 + w["bigram"][(28 + 6) % 10])
    y = P.embed([9], {"scale": 0.5, "bigram": bigram}, w, memory)
    assert torch.allclose(y[0], w["embed"][9] * 0.5 + w["bigram"][(14 + 27) % 10])


def test_plain_recurrence_is_its_unrolled_sum():
    """o_t = sum_{s <= t} (q_t * prod_{s < u <= t} a_u) . k_s v_s."""
    T, d, dv = 9, 4, 3
    q, k, v = randn(T, d), randn(T, d, seed=1), randn(T, dv, seed=2)
    a = torch.sigmoid(randn(T, d, seed=3))
    out, _ = P.gla_scan(q, k, v, a, torch.zeros(d, dv, dtype=F64))
    for t in range(T):
        want = sum(((q[t] * a[s + 1:t + 1].prod(dim=0)) @ k[s]) * v[s] for s in range(t + 1))
        assert torch.allclose(out[t], want)


def test_plain_rotation_pairs_neighbours():
    x = torch.zeros(1, 6, dtype=F64)
    x[0, 2] = 1.0                                  # the first of the second pair
    y = P.rotate_pairs(x, torch.tensor([3]), 4, 100.0)
    a = 3 * 100.0 ** -0.5
    assert torch.allclose(y[0], torch.tensor([0, 0, torch.cos(torch.tensor(a, dtype=F64)), torch.sin(torch.tensor(a, dtype=F64)), 0, 0], dtype=F64))
    x[0, 5] = 2.0
    assert P.rotate_pairs(x, torch.tensor([3]), 4, 100.0)[0, 5] == 2.0        # behind dims: as it is


def test_plain_choice_inside_groups():
    """Four groups of two; corrections make the choice and not the weights; a group outside the kept ones gives nothing,
    also where every choice score is negative."""
    z = torch.tensor([[2.0, -3.0, 0.5, 0.4, -1.0, -1.0, 1.9, 0.0]], dtype=F64)
    w = {"router": torch.eye(8, dtype=F64), "correction": torch.tensor([-2.0, -2.0, -1.0, -1.0, -3.0, -3.0, -1.9, -1.0], dtype=F64)}
    router = {"experts": 8, "top": 3, "scale": 2.0, "groups": {"count": 4, "keep": 2}}
    s = torch.sigmoid(z)[0]
    c = s + w["correction"]
    groups = sorted(range(4), key=lambda g: -float(c[2 * g] + c[2 * g + 1]))[:2]
    allowed = [e for e in range(8) if e // 2 in groups]
    want = sorted(allowed, key=lambda e: -float(c[e]))[:3]
    chosen, weight = P.route(z, router, w, "")
    assert chosen[0].tolist() == want and float(c.max()) < 0
    assert torch.allclose(weight[0], s[want] / s[want].sum() * 2.0) and abs(float(weight.sum()) - 2.0) < 1e-12


def test_plain_attention_runs_in_the_latent_space():
    """Scores and values made from the latent vectors (W_uk on the query, W_uv behind the mix) give the same result."""
    m = GC.latent(3, 5, 4, 6, 7, 8, 0.3)
    w = {n: randn(*s, seed=i) for i, (n, s) in enumerate({"dq": (7, 11), "dq.norm": (7,), "uq": (27, 7), "dkv": (12, 11), "dkv.norm": (8,),
                                                          "uk": (15, 8), "uv": (18, 8), "o": (11, 18)}.items())}
    h, pos = randn(10, 11, seed=50), torch.arange(10)
    kept = P.latent_keys(h, pos, m, w, "", 1e-5)
    want = P.latent_attention(h, pos, m, w, "", 1e-5, kept)
    q, q_rot = P.latent_queries(h, pos, m, w, "", 1e-5)
    ql = torch.einsum("thd,hdr->thr", q, w["uk"].reshape(3, 5, 8))
    score = (torch.einsum("thr,sr->hts", ql, kept[0]) + torch.einsum("thd,sd->hts", q_rot, kept[1])) * 0.3
    score = score.masked_fill(torch.ones(10, 10, dtype=torch.bool).triu(1), float("-inf"))
    mix = torch.einsum("hts,sr->thr", torch.softmax(score, -1), kept[0])
    assert torch.allclose(torch.einsum("thr,hvr->thv", mix, w["uv"].reshape(3, 6, 8)).reshape(10, 18) @ w["o"].T, want)


def test_the_measured_configurations_are_valid():
    """bench.py --design gemepel builds these."""
    import os
    import sys
    sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
    import bench
    from yalm_amd.config import config_from_dict
    for width in (2048, 4096):
        cfg = config_from_dict(bench.gemepel_config(width))
        spec = cfg.to_spec()
        assert {l["type"] for l in cfg.layers} == {"latent_attention", "gla"}
        assert [e.writes_cache for e in spec.schedule].count(False) == 1
