"""The Pamazen configuration reader and model spec on the CPU, pins of the plain implementation, and the cache group that
keeps a request's first positions."""
import copy
import math

import pytest
import torch

import pamazen_models as PM
import plain_pamazen as PP
from infernum_amd import models  # noqa: F401  (registers the architectures)
from infernum_amd.cache import CacheConfig, CacheManager
from infernum_amd.config.base import ConfigError
from infernum_amd.config.pamazen import PamazenConfig
from infernum_amd.config.registry import config_from_dict, model_spec_for
from infernum_amd.models.model import DecoderModel
from infernum_amd.parts.base import CacheSpec, Runtime
from infernum_amd.weights.safetensors_io import open_model_tensors

CPU = Runtime(torch.device("cpu"), torch.float32)
F64 = torch.float64


@pytest.mark.parametrize("name", list(PM.RAW))
def test_reads_every_key_and_writes_it_back(name):
    raw = PM.RAW[name]
    cfg = config_from_dict(raw)
    assert isinstance(cfg, PamazenConfig) and cfg.to_dict() == raw
    assert (cfg.vocab_size, cfg.hidden_size, cfg.num_hidden_layers) == (raw["vocab"], raw["width"], len(raw["layers"]))
    without = copy.deepcopy(raw)
    without.pop("residual_mult")
    assert config_from_dict(without).residual_mult == 1.0


@pytest.mark.parametrize("name", list(PM.RAW))
def test_the_spec_wants_the_tensors_of_the_file(name):
    raw = PM.RAW[name]
    ranked = copy.deepcopy(raw)
    for layer in ranked["layers"]:
        if layer["type"] == "parallel":
            layer["mixer"]["right"]["rank"] = 12
    assert config_from_dict(ranked).to_dict() == ranked
    spec = model_spec_for(config_from_dict(ranked))
    expected = DecoderModel(spec, CPU).expected_weights()
    want = {k: tuple(v.shape) for k, v in expected.items() if v.write_when_random}
    have = PP.tensor_shapes(raw, 12)
    spare = set(have) - set(want)                 # the number of the first layer that mixes values is not read
    assert spare == {f"l{i}.mix.vmix" for i in [config_from_dict(raw).first_value_layer] if i is not None}
    assert spare <= set(spec.ignored_tensors) and want == {k: v for k, v in have.items() if k not in spare}
    # a file's own middle of the decays is taken as it is
    assert all(-1 in ws.shape for n, ws in DecoderModel(model_spec_for(config_from_dict(raw)), CPU).expected_weights().items()
               if n.endswith((".w1", ".w2")))
    assert all(l.block == "hyper" for l in spec.layers)
    last = [p for l in spec.layers for _, p in l.extra.values() if p.params["last"]]
    tail = spec.layers[-1]
    assert last == [tail.extra["feed_forward_hyper" if tail.feed_forward is not None else "mixer_hyper"][1]]


def test_what_every_mixer_keeps():
    model = DecoderModel(model_spec_for(config_from_dict(PM.P1)), CPU)
    needs = model.cache_needs()
    # a side-by-side layer keeps nothing itself; its two mixers have pages and a state of their own
    assert needs[0] == (None, None)
    assert needs[1][0] == CacheSpec("window", 2, 32, 20, keep_first=3) and needs[1][1] is None
    assert needs[2][0] is None and needs[2][1].shape == (3 * 16 * 16,)
    assert needs[3][0].kind == "full" and {t.name: t.shape for t in needs[3][0].payload} == {"k": (2, 32), "v": (2, 16)}
    assert needs[1][0].group_key() != CacheSpec("window", 2, 32, 20).group_key()


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0].__setitem__("type", "conv"), "type"),
    (lambda c: c["layers"][0]["mixer"]["left"].__setitem__("kv_heads", 4), "multiple"),
    (lambda c: c["layers"][0]["mixer"]["left"].__setitem__("vdim", 16), "vdim"),
    (lambda c: c["layers"][0]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("dims", 7), "even"),
    (lambda c: c["layers"][1]["mixer"].__setitem__("vdim", 48), "mix"),
    (lambda c: c["layers"][0]["mlp"].__setitem__("kind", "dense"), "kind"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].__setitem__("count", 3), "groups"),
    (lambda c: c["layers"][0]["mlp"]["router"].__setitem__("top", 5), "groups"),
    (lambda c: c.pop("norm"), "norm"),
    (lambda c: c.pop("streams"), "streams"),
])
def test_a_wrong_configuration_is_refused(change, message):
    raw = copy.deepcopy(PM.P1)
    change(raw)
    with pytest.raises(ConfigError, match=message):
        config_from_dict(raw)


def test_model_folder_round_trip(tmp_path):
    cfg, w = PM.write_model("P2", str(tmp_path))
    found = open_model_tensors(str(tmp_path))
    assert set(found) == set(w) and config_from_dict(cfg).first_value_layer == 2


# ------------------------------------------------------------------------------------- the cache
@pytest.mark.parametrize("ps,window,keep", [(4, 7, 5), (16, 20, 3), (4, 1, 17), (8, 30, 8), (4, 6, 0), (16, 5, 100)])
def test_a_window_group_keeps_the_first_pages(ps, window, keep):
    cache = CacheManager([(CacheSpec("window", 1, 4, window, keep_first=keep), None)], [None], CacheConfig(page_size=ps, num_pages=60))
    for req, sizes in (("a", [3, 9, 1, 1, 20, 2] + [1] * 40), ("b", [50, 7])):
        assert cache.admit(req)
        n = 0
        for k in sizes:
            assert cache.reserve(req, k)
            cache.commit(req, k)
            n += k
            pages = cache.block_table(0, req).pages
            for i, page in enumerate(pages):
                positions = range(i * ps, (i + 1) * ps)
                # needed: a position that the next query (at n) or a later one sees
                needed = any(p < keep or p > n - window for p in positions)
                assert (page >= 0) == needed, (n, i)
            cache.check()
    assert len(cache.block_table(0, "a").live_pages()) == sum(p >= 0 for p in cache.block_table(0, "a").pages)
    for req in ("a", "b"):
        cache.release(req)
        cache.check()
    assert cache.free_pages(0) == 60


# ------------------------------------------------------------------------------------- pins of the plain model
def test_plain_mask_by_brute_force():
    seen = PP.seen_keys(15, 4, 2)
    for i in range(15):
        for j in range(15):
            assert bool(seen[i, j]) == (j <= i and (i - j < 4 or j < 2))
    assert torch.equal(PP.seen_keys(6), torch.ones(6, 6, dtype=torch.bool).tril())


def test_plain_softmax_with_one_added_and_with_a_sink():
    torch.manual_seed(1)
    s = torch.randn(6, 6, dtype=F64)
    for sink in (0.0, 0.7, -1e9):
        w = PP.sink_softmax(s, PP.seen_keys(6), torch.tensor(sink, dtype=F64))
        for i in range(6):
            e = s[i, :i + 1].exp()
            assert torch.allclose(w[i, :i + 1], e / (e.sum() + math.exp(sink))) and w[i, i + 1:].abs().sum() == 0


def test_plain_rotation_of_neighbours():
    x = torch.arange(6, dtype=F64).view(1, 1, 6) + 1
    ang = PP.rotation_angles(torch.tensor([3]), 4, 100.0, 2.0)
    assert torch.allclose(ang, torch.tensor([[1.5, 3 * 100.0 ** -0.5 / 2.0]], dtype=F64))
    y = PP.rotate_pairs(x, ang, 4)
    c, s = torch.cos(ang[0]), torch.sin(ang[0])
    assert torch.allclose(y[0, 0], torch.stack([1 * c[0] - 2 * s[0], 2 * c[0] + 1 * s[0], 3 * c[1] - 4 * s[1], 4 * c[1] + 3 * s[1],
                                               x[0, 0, 4], x[0, 0, 5]]))


def test_plain_delta_rule():
    torch.manual_seed(2)
    T, d = 7, 3
    r, k, v = (torch.randn(T, d, dtype=F64) for _ in range(3))
    w, a = torch.rand(T, d, dtype=F64), torch.rand(T, d, dtype=F64)
    o, S = PP.delta_recurrence(r, k, v, w, a)
    want = torch.zeros(d, d, dtype=F64)
    u = k / torch.sqrt((k * k).sum(1, keepdim=True) + 1e-6)
    for t in range(T):
        old = want.clone()
        for i in range(d):
            for j in range(d):
                want[i, j] = w[t, i] * old[i, j] - a[t, i] * u[t, i] * sum(u[t, m] * old[m, j] for m in range(d)) + k[t, i] * v[t, j]
        assert torch.allclose(o[t], want.T @ r[t])
    assert torch.allclose(S, want)
    o1, S1 = PP.delta_recurrence(r[:4], k[:4], v[:4], w[:4], a[:4])
    o2, S2 = PP.delta_recurrence(r[4:], k[4:], v[4:], w[4:], a[4:], S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)
    # nothing decays and everything along the key is taken out: a key written again replaces what it wrote
    one = torch.ones(2, d, dtype=F64)
    kk = torch.tensor([[0.0, 2.0, 0.0]] * 2, dtype=F64)
    vv = torch.tensor([[1.0, 2.0, 3.0], [4.0, 5.0, 6.0]], dtype=F64)
    _, S = PP.delta_recurrence(kk, kk, vv, one, one)
    assert torch.allclose(S[1], 2.0 * vv[1], atol=1e-5)


def test_plain_choice_of_experts():
    s = torch.tensor([[0.1, 0.2, 0.3, 0.05, 0.25, 0.1]], dtype=F64)
    zero = torch.zeros(6, dtype=F64)
    ids, wts = PP.choose_experts(s, zero, 2, 1, 1)
    assert ids.tolist() == [[2, 4]] and torch.allclose(wts, torch.tensor([[0.3, 0.25]], dtype=F64))
    # three groups of two, one kept: group 1 has the largest score, and its second expert the smallest of all
    ids, wts = PP.choose_experts(s, zero, 2, 3, 1)
    assert ids.tolist() == [[2, 3]] and torch.allclose(wts, torch.tensor([[0.3, 0.05]], dtype=F64))
    # choice scores below zero stay choosable inside a kept group, and the weights do not see the correction
    corr = torch.tensor([-5.0, -5.0, -6.0, -6.0, -1.0, -1.1], dtype=F64)
    ids, wts = PP.choose_experts(s, corr, 2, 3, 1)
    assert ids.tolist() == [[4, 5]] and torch.allclose(wts, torch.tensor([[0.25, 0.1]], dtype=F64))
    assert float(PP.choice_margin(s, zero, 2, 1, 1)) == pytest.approx(0.05)


def test_plain_streams_mix_from_the_old_ones():
    torch.manual_seed(3)
    X, y = torch.randn(3, 4, 5, dtype=F64), torch.randn(4, 5, dtype=F64)
    mix, b = torch.randn(3, 3, dtype=F64), torch.randn(3, dtype=F64)
    new = PP.hyper_write(X, y, mix, b, 0.5)
    for t in range(3):
        assert torch.allclose(new[t], sum(mix[s, t] * X[s] for s in range(3)) + 0.5 * b[t] * y)
    assert torch.allclose(PP.hyper_read(X, b), sum(b[s] * X[s] for s in range(3)))


@pytest.mark.parametrize("name", ["P1", "P3"])
def test_plain_model_is_causal_and_every_kept_position_counts(name):
    cfg = PM.RAW[name]
    w = PP.random_weights(cfg, 3)
    toks = torch.randint(0, cfg["vocab"], (30,), generator=torch.Generator().manual_seed(4)).tolist()
    a = PP.forward(cfg, w, toks)
    assert torch.allclose(a[:20], PP.forward(cfg, w, toks[:20]))
    other = copy.deepcopy(cfg)
    for layer in other["layers"]:
        if layer["type"] == "parallel" and layer["mixer"]["left"].get("mask"):
            layer["mixer"]["left"]["mask"]["keep_first"] = 0
    assert (PP.forward(other, w, toks) - a)[-1].abs().max() > 1e-3
