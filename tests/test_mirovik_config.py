"""The Mirovik configuration reader and model spec on the CPU, the bias tables' rows, and pins of the plain implementation."""
import copy
import math

import pytest
import torch

import mirovik_models as MM
import plain_mirovik as MP
from infernum_amd import models  # noqa: F401  (registers the architectures)
from infernum_amd.config.base import ConfigError
from infernum_amd.config.mirovik import MirovikConfig
from infernum_amd.config.registry import config_from_dict, model_spec_for
from infernum_amd.kernels.api import DISTANCE_PAD, distance_table
from infernum_amd.models.model import DecoderModel
from infernum_amd.parts.base import Runtime
from infernum_amd.parts.softmax_attention import bias_by_distance, bucket_starts
from infernum_amd.weights.safetensors_io import open_model_tensors

CPU = Runtime(torch.device("cpu"), torch.float32)
F64 = torch.float64


@pytest.mark.parametrize("name", list(MM.RAW))
def test_reads_every_key_and_writes_it_back(name):
    raw = MM.RAW[name]
    cfg = config_from_dict(raw)
    assert isinstance(cfg, MirovikConfig) and cfg.to_dict() == raw
    assert (cfg.vocab_size, cfg.hidden_size, cfg.num_hidden_layers) == (raw["vocab"], raw["width"], len(raw["layers"]))
    assert [i for i, _ in cfg.layer_runs()] == [i for i, _ in MP.layer_runs(raw)]
    without = copy.deepcopy(raw)
    without.pop("embedding")
    assert config_from_dict(without).embedding_scale == 1.0


@pytest.mark.parametrize("name", list(MM.RAW))
def test_the_spec_wants_the_tensors_of_the_file(name):
    raw = MM.RAW[name]
    spec = model_spec_for(config_from_dict(raw))
    expected = DecoderModel(spec, CPU).expected_weights()
    want = {k: tuple(v.shape) for k, v in expected.items() if v.write_when_random}
    assert want == MP.tensor_shapes(raw)
    assert expected["head"].fallback == "embed"               # the head is the embedding table
    # a file's own bias tables are taken as they are
    bare = copy.deepcopy(raw)
    for layer in bare["layers"]:
        if layer["type"] == "parallel":
            layer["mixer"]["left"].pop("buckets")
    shapes = {n: ws.shape for n, ws in DecoderModel(model_spec_for(config_from_dict(bare)), CPU).expected_weights().items()}
    assert all(s[0] == -1 for n, s in shapes.items() if n.endswith(".rel"))
    assert all(l.block == "sandwich" for l in spec.layers)
    enters = [i for i, l in enumerate(spec.layers) if "stream_in" in l.extra]
    assert enters == ([raw["loop"]["start"]] if raw.get("loop") else [])


def test_what_every_mixer_keeps_in_every_pass():
    model = DecoderModel(model_spec_for(config_from_dict(MM.V1)), CPU)
    needs = model.cache_needs()
    # layer 0; then twice: layer 1 (nothing itself, pages, a state) and layer 2; then layer 3
    mamba = [n[1].shape for n in needs if n[0] is None and n[1] is not None]
    assert mamba == [(3 * 96 + 16 * 96,), (3 * 16 * 32,), (2 * 128 + 8 * 128,), (3 * 16 * 32,), (2 * 128 + 8 * 128,), (2 * 32 * 16,)]
    pages = [{t.name: t.shape for t in n[0].payload} for n in needs if n[0] is not None and n[0].payload]
    assert pages == [{"k": (2, 32), "v": (2, 16)}] * 2 + [{"k": (3, 16), "v": (3, 16)}]
    assert sum(n[0] is not None for n in needs) == 3 and all(n[0].kind == "full" for n in needs if n[0] is not None)
    assert [e.pass_index for e in model.spec.schedule] == [0, 0, 0, 1, 1, 0]


@pytest.mark.parametrize("change, message", [
    (lambda c: c["layers"][0].__setitem__("type", "conv"), "type"),
    (lambda c: c["layers"][1]["mixer"]["left"].__setitem__("kv_heads", 3), "multiple"),
    (lambda c: c["layers"][1]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][1]["mixer"]["right"].__setitem__("decay", [0.5]), "decay"),
    (lambda c: c["layers"][1]["mixer"]["right"].__setitem__("decay", [0.5, 0.5, 1.5]), "decay"),
    (lambda c: c["layers"][1]["mixer"]["right"]["rot"].__setitem__("dims", 7), "even"),
    (lambda c: c["layers"][1]["mixer"]["right"]["rot"].__setitem__("dims", 18), "at most"),
    (lambda c: c["layers"][1]["mixer"]["left"].pop("bias_max"), "bias_max"),
    (lambda c: c["layers"][0]["mixer"].pop("dt_rank"), "dt_rank"),
    (lambda c: c["layers"][0]["mlp"].__setitem__("kind", "sparse"), "kind"),
    (lambda c: c["layers"][0]["mlp"]["router"].__setitem__("top", 7), "experts"),
    (lambda c: c["loop"].__setitem__("stop", 5), "loop"),
    (lambda c: c.pop("norm"), "norm"),
])
def test_a_wrong_configuration_is_refused(change, message):
    raw = copy.deepcopy(MM.V1)
    change(raw)
    with pytest.raises(ConfigError, match=message):
        config_from_dict(raw)


def test_model_folder_round_trip(tmp_path):
    cfg, w = MM.write_model("V2", str(tmp_path))
    assert set(open_model_tensors(str(tmp_path))) == set(w)
    assert config_from_dict(cfg).to_dict() == cfg


# ------------------------------------------------------------------------------------- the bias by distance
@pytest.mark.parametrize("rows,far", [(2, 3), (4, 5), (6, 9.5), (10, 50), (14, 30), (16, 256), (20, 40), (32, 128), (32, 2048), (64, 300), (48, 25)])
def test_rows_of_the_bias_table(rows, far):
    """Against the plain rule in whole numbers for every distance, and against its logarithms wherever those are not
    within rounding of a whole number."""
    starts, h = bucket_starts(rows, far), rows // 2
    assert len(starts) == rows and starts[:h] == list(range(h)) and all(b >= a for a, b in zip(starts, starts[1:]))
    close = 0
    for n in range(int(2 * far) + 5):
        row = max(k for k, s in enumerate(starts) if s <= n)
        assert row == MP.bucket_of(n, rows, far), n
        if n >= h:
            x = math.log(n / h) / math.log(far / h) * (rows - h)
            if abs(x - round(x)) < 1e-9:
                close += 1
            else:
                assert row == min(rows - 1, h + math.floor(x)), n
        else:
            assert row == n
    assert close >= 1                               # n = h at the least


def test_bias_table_by_distance_and_backwards():
    rel = torch.arange(12, dtype=torch.float32).view(6, 2)
    by = bias_by_distance(rel, 9.5)
    assert by.shape[0] == 2 and by[0].tolist() == [2.0 * MP.bucket_of(n, 6, 9.5) for n in range(by.shape[1])]
    assert by[0, -1] == 10.0 and by[0, -2] < 10.0            # it ends with the first distance of the last row
    t = distance_table(by)
    span = by.shape[1]
    assert t.shape == (2, span + 2 * DISTANCE_PAD) and t.is_contiguous()
    for n in range(span):
        assert t[1, DISTANCE_PAD + span - 1 - n] == by[1, n]
    assert (t[1, :DISTANCE_PAD] == by[1, -1]).all() and (t[:, DISTANCE_PAD + span:] == 0).all()
    for rows, far in ((2, 1.0), (8, 4), (8, 3)):
        with pytest.raises(ValueError, match="furthest"):
            bucket_starts(rows, far)


# ------------------------------------------------------------------------------------- pins of the plain model
def test_plain_attention_by_brute_force():
    torch.manual_seed(1)
    T, H, G, d, dv = 9, 4, 2, 3, 2
    q, k, v = torch.randn(T, H, d, dtype=F64), torch.randn(T, G, d, dtype=F64), torch.randn(T, G, dv, dtype=F64)
    rel = torch.randn(4, H, dtype=F64)
    o = MP.biased_attention(q, k, v, 0.7, MP.distance_bias(T, rel, 6.0)).view(T, H, dv)
    bucket = [0, 1, 2, 2, 3, 3, 3, 3, 3]                 # 2 + floor(2 ln(n / 2) / ln 3), at most 3
    for i in range(T):
        for h in range(H):
            s = [0.7 * float(q[i, h] @ k[j, h // 2]) + float(rel[bucket[i - j], h]) for j in range(i + 1)]
            e = [math.exp(x) for x in s]
            want = sum(x * v[j, h // 2] for j, x in enumerate(e)) / sum(e)
            assert torch.allclose(o[i, h], want)


def test_plain_rotation_of_halves():
    x = (torch.arange(6, dtype=F64) + 1).view(1, 1, 6)
    y = MP.rotate_half(x, torch.tensor([3]), 4, 100.0)[0, 0]
    a, b = 3.0, 3.0 * 100.0 ** -0.5
    want = [1 * math.cos(a) - 3 * math.sin(a), 2 * math.cos(b) - 4 * math.sin(b), 3 * math.cos(a) + 1 * math.sin(a),
            4 * math.cos(b) + 2 * math.sin(b), 5, 6]
    assert torch.allclose(y, torch.tensor(want, dtype=F64))


def test_plain_recurrences_by_brute_force():
    torch.manual_seed(2)
    T = 7
    q, k, v = torch.randn(T, 3, dtype=F64), torch.randn(T, 3, dtype=F64), torch.randn(T, 2, dtype=F64)
    o, S = MP.retention(q, k, v, 0.7)
    for t in range(T):
        assert torch.allclose(o[t], sum(0.7 ** (t - j) * (q[t] @ k[j]) * v[j] for j in range(t + 1)))
    o1, S1 = MP.retention(q[:4], k[:4], v[:4], 0.7)
    o2, S2 = MP.retention(q[4:], k[4:], v[4:], 0.7, S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)
    x, dt, A = torch.randn(T, 2, dtype=F64), torch.rand(T, 2, dtype=F64), -torch.rand(2, 3, dtype=F64)
    B, C, D = torch.randn(T, 3, dtype=F64), torch.randn(T, 3, dtype=F64), torch.randn(2, dtype=F64)
    y, S = MP.selective_scan(x, dt, A, B, C, D)
    for c in range(2):
        for t in range(T):
            want = D[c] * x[t, c]
            for j in range(t + 1):
                for n in range(3):
                    want = want + torch.exp(A[c, n] * dt[j + 1:t + 1, c].sum()) * dt[j, c] * x[j, c] * B[j, n] * C[t, n]
            assert torch.allclose(y[t, c], want)
    y1, S1 = MP.selective_scan(x[:3], dt[:3], A, B[:3], C[:3], D)
    y2, S2 = MP.selective_scan(x[3:], dt[3:], A, B[3:], C[3:], D, S1)
    assert torch.allclose(torch.cat([y1, y2]), y) and torch.allclose(S2, S)


def test_plain_convolution_and_experts():
    x = torch.tensor([[1.0], [2.0], [3.0]], dtype=F64)
    y = MP.causal_conv(x, torch.tensor([[0.5, 10.0]], dtype=F64), torch.tensor([0.25], dtype=F64))
    assert y.flatten().tolist() == [10.25, 20.75, 31.25]
    torch.manual_seed(3)
    m = MM._moe(4, 3, 2, 5)
    w = {k[4:]: t.to(F64) for k, t in ((k[3:], t) for k, t in MP.random_weights(
        {"vocab": 4, "width": 6, "layers": [MM._layer("mamba1", MM._mamba(2, 1, 1, 1), m)]}, 1).items()) if k.startswith("mlp.")}
    f = torch.randn(5, 6, dtype=F64)
    out = MP.routed_experts(f, w, "", m)
    for n in range(5):
        s = 1 / (1 + torch.exp(-(w["router"] @ f[n])))
        want = MP.gated_expert(f[n:n + 1], w, "shared.")[0]
        for e in s.argsort(descending=True)[:2].tolist():
            want = want + MP.gated_expert((s[e] * f[n])[None], w, f"e{e}.")[0]
        assert torch.allclose(out[n], want)


@pytest.mark.parametrize("name", ["V1", "V3", "V4"])
def test_plain_model_is_causal_and_every_pass_counts(name):
    cfg = MM.RAW[name]
    w = MP.random_weights(cfg, 3)
    toks = torch.randint(0, cfg["vocab"], (24,), generator=torch.Generator().manual_seed(4)).tolist()
    a = MP.forward(cfg, w, toks)
    assert torch.allclose(a[:15], MP.forward(cfg, w, toks[:15]))
    for t in range(cfg["loop"]["times"]):
        other = dict(w)
        other["loop.step"] = w["loop.step"].clone()
        other["loop.step"][t] = 0
        assert (MP.forward(cfg, other, toks) - a).abs().max() > 1e-3


@pytest.mark.parametrize("name", list(MM.RAW))
def test_decided_routers_have_wide_margins(name):
    cfg = MM.RAW[name]
    w = MM.decided(cfg, MP.random_weights(cfg, MM.SEED[name]))
    toks = torch.randint(0, cfg["vocab"], (60,), generator=torch.Generator().manual_seed(5)).tolist()
    margins = []
    MP.forward(cfg, w, toks, margins=margins)
    assert not margins or min(float(m.min()) for m in margins) > 0.01
