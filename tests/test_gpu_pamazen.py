"""The Pamazen decoder on the GPU against the plain implementation (plain_pamazen.py): each mechanism alone, then the
engine on small models of other sizes than any real one: whole prompts, the tail decoded token by token, portions down
to two tokens, mixed batches over pools so small that pages and state slots are used again (freed pages hold NaN), a key
that stands out just inside and just outside a window and among the first positions and the next ones, far back among
hundreds, a state that reaches hundreds of tokens back, long decoding from graphs, and greedy generation through the
runtime and its scheduler."""
import math

import pytest
import torch

import pamazen_models as PM
import plain_pamazen as PP
import trace_tools as TT
from part_harness import DEV, TOL as PART_TOL, Steps, build, dense, rel_err, runtime

pytestmark = pytest.mark.gpu
BOTH = pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
# largest |difference| of a logit as a fraction of the RMS of the plain logits
TOL = {"float32": 3e-5, "bfloat16": 6e-2}
NAMES = ["P1", "P2", "P3", "P4", "P5"]
LENGTHS = {"P1": (1, 7, 45, 83, 130), "P2": (3, 61, 33, 97), "P3": (9, 70, 121), "P4": (2, 17, 64, 150), "P5": (1, 64, 65, 140)}
MIXED = {"P1": (70, 131, 64, 150, 33, 97, 66, 81), "P2": (150, 165, 120, 190, 147), "P3": (129, 65, 90, 47, 72, 99),
         "P4": (70, 131, 64, 150, 33, 97), "P5": (150, 100, 64, 190, 129, 77)}
PAGE = {"P1": 16, "P2": 4, "P3": 8, "P4": 16, "P5": 12}
EPS = 1e-5


def _x(n, h, dtype, seed=0, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    x = torch.randn(n, h, generator=g) * scale
    return x.to(torch.bfloat16).float() if dtype == "bfloat16" else x


def _tol(dtype, want, rounded):
    """Three times what rounding every stored activation to bfloat16 costs the plain form, and at least the parts'
    usual tolerance; in 32-bit the parts' usual one."""
    if dtype != "bfloat16":
        return PART_TOL[dtype]
    return max(PART_TOL[dtype], 3.0 * rel_err(rounded().to(torch.bfloat16), want))


def _layer_weights(layer, W, seed, rank=12):
    cfg = {"vocab": 4, "width": W, "streams": 1, "layers": [layer]}
    return {k[3:]: v.double() for k, v in PP.random_weights(cfg, seed, rank=rank).items() if k.startswith("l0.")}


def _mixer_weights(kind, m, W, seed, prefix="mix.", rank=12):
    w = _layer_weights({"type": kind, "mixer": m, "mlp": None}, W, seed, rank)
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def _rope(rot, head_dim):
    if not rot:
        return {"kind": "none"}
    factor = (rot.get("scaling") or {}).get("factor")
    return {"kind": "rope", "params": {"head_dim": head_dim, "theta": rot["base"], "rotary_dim": rot["dims"],
                                       "scaling": {"rope_type": "linear", "factor": factor} if factor else None,
                                       "pairing": "neighbours"}}


def _att_params(m, W, mix=None):
    return {"hidden_size": W, "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "head_dim": m["dim"],
            "value_dim": m["vdim"], "scale": m["scale"], "position": _rope(m.get("rot"), m["dim"]), "sink": "zero",
            "value_mix": mix}


def _left_params(m, W):
    mask = m.get("mask") or {}
    return {"hidden_size": W, "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "head_dim": m["dim"],
            "value_dim": m["dim"], "scale": m["scale"], "window": mask.get("size"), "keep_first": mask.get("keep_first", 0),
            "softcap": m.get("softcap"), "sink": "learned", "qk_norm": True, "norm_eps": EPS, "values": "keys"}


def _delta_params(m, W):
    return {"hidden_size": W, "num_heads": m["heads"], "head_dim": m["dim"], "norm_eps": EPS}


def _side_params(m, W):
    return {"hidden_size": W, "mixers": {
        "left": {"kind": "softmax_attention", "scale": m["left_scale"], "params": _left_params(m["left"], W)},
        "right": {"kind": "delta_rule", "scale": m["right_scale"], "params": _delta_params(m["right"], W)}}}


def _build(kind, params, rt, tensors):
    """A mixer with all its tensors given (the sizes that it reads off them among them)."""
    from infernum_amd.parts import PartSpec, make_part
    part = make_part("mixer", PartSpec(kind, params), rt)
    w = {n: t.to(torch.float32) for n, t in tensors.items()}
    if rt.dtype == torch.bfloat16:
        w = {n: t.to(torch.bfloat16).float() for n, t in w.items()}
    part.load({n: w[n].to(DEV).to(rt.dtype if ws.follows_compute_dtype or rt.is_fp32 else torch.float32)
               for n, ws in part.weights().items()})
    return part, {n: t.double() for n, t in w.items()}


def _steps_for(mixer, rt, page_size, num_pages, slots=4, poison=True):
    needs, names = [(mixer.cache_spec(), mixer.state_spec())], []
    for name, part in getattr(mixer, "cached_companions", lambda: {})().items():
        needs.append((part.cache_spec(), part.state_spec()))
        names.append(name)
    steps = Steps(needs, rt, page_size=page_size, num_pages=num_pages, slots=slots, poison=poison)
    steps.views[0].others = {n: steps.views[1 + i] for i, n in enumerate(names)}
    return steps


def _run_mixer(mixer, steps, x, cuts, rt, request="a"):
    """Feeds x [T, W] of one request through the mixer in the portions ``cuts``."""
    out, p = [], 0
    for n in cuts:
        ctx, packed = steps.begin([(request, n)])
        out.append(dense(mixer.forward(x[p:p + n].to(DEV).to(rt.dtype), ctx, steps.views[0]), rt).float().cpu())
        steps.end(packed)
        p += n
    assert p == x.shape[0]
    return torch.cat(out)


def CUTS(T):
    return [[c for c in cuts if c > 0] for cuts in
            ([T], [1] * T, [T - 9] + [1] * 9, [2] * (T // 2) + [T % 2], [7, 2, 13, 2, 3, T - 27])]


# ------------------------------------------------------------------------------------ small kernels alone
@BOTH
@pytest.mark.parametrize("S,H,N", [(1, 64, 3), (3, 100, 17), (4, 1028, 5), (2, 30, 9), (5, 2052, 3), (8, 7000, 2), (9, 48, 11), (17, 26, 4),
                                   (3, 9001, 2)])
def test_streams_written_back_read_and_closed(dtype, S, H, N):
    """The three forms of the step between sublayers: entering from one stream that all are copies of; writing back a
    result (a tensor, or partial sums) and entering the next; closing with the sum."""
    from infernum_amd.kernels import api as K
    rt = runtime(dtype)
    g = torch.Generator().manual_seed(S)
    rnd = lambda *s: torch.randn(*s, generator=g)                # noqa: E731
    h, mix, out_w, in_w, norm = rnd(N, H), rnd(S, S), rnd(S), rnd(S), rnd(H)
    y = [rnd(N, H) for _ in range(3)]
    dev = lambda t: t.to(torch.float32).contiguous().to(DEV)     # noqa: E731
    X = h.double()[None].repeat(S, 1, 1)
    x = torch.empty((N, H), dtype=rt.dtype, device=DEV)
    K.hyper_step(dev(h), S, None, None, None, None, dev(in_w), dev(norm), EPS, x)
    want = PP.unit_rms(PP.hyper_read(X, in_w.double()), EPS) * norm.double()
    assert rel_err(x, want) <= PART_TOL[dtype]
    # the first result: the streams begin to exist
    delta = y[0].to(rt.dtype)
    new = torch.empty((N, S, H), dtype=torch.float32, device=DEV)
    K.hyper_step(dev(h), S, new, delta.to(DEV), dev(mix), dev(out_w), dev(in_w), dev(norm), EPS, x)
    X = PP.hyper_write(X, delta.double(), mix.double(), out_w.double(), 1.0)
    assert rel_err(new.permute(1, 0, 2).cpu(), X) <= 1e-5
    assert rel_err(x, PP.unit_rms(PP.hyper_read(X, in_w.double()), EPS) * norm.double()) <= PART_TOL[dtype]
    # a second one, as partial sums, in place
    parts = K.SplitSum(torch.stack([dev(t) for t in y]))
    K.hyper_step(new, S, new, parts, dev(mix), dev(out_w), dev(in_w), dev(norm), EPS, x)
    X = PP.hyper_write(X, sum(t.double() for t in y), mix.double(), out_w.double(), 1.0)
    assert rel_err(new.permute(1, 0, 2).cpu(), X) <= 1e-5
    assert rel_err(x, PP.unit_rms(PP.hyper_read(X, in_w.double()), EPS) * norm.double()) <= PART_TOL[dtype]
    # the last: the sum, the streams left as they are
    total, before = torch.empty((N, H), dtype=torch.float32, device=DEV), new.clone()
    K.hyper_step(new, S, None, delta.to(DEV), dev(mix), dev(out_w), None, None, 0.0, total)
    assert torch.equal(new, before)
    assert rel_err(total, PP.hyper_write(X, delta.double(), mix.double(), out_w.double(), 1.0).sum(0)) <= 1e-5


@BOTH
@pytest.mark.parametrize("nh,nkv,d,dv,rot,ps,N,keys", [(4, 2, 32, 16, 16, 16, 37, False), (3, 3, 12, 10, 6, 4, 9, False), (6, 2, 32, 32, 0, 8, 40, True),
                                                      (2, 1, 64, 128, 64, 12, 130, False), (5, 5, 20, 20, 0, 4, 7, True), (1, 1, 16, 8, 2, 4, 1, False)])
def test_rows_into_queries_keys_and_values(dtype, nh, nkv, d, dv, rot, ps, N, keys):
    """Norms, rotation of neighbours, the values' own size, their factor and their mixture with another layer's rows
    (columns of wider rows), each value at its token's place of the transposed page."""
    from infernum_amd.kernels import api as K
    rt = runtime(dtype)
    row = (nh + nkv) * d + (0 if keys else nkv * dv)
    x = _x(N, row + 8, dtype, 3)
    first = _x(N, nkv * dv + 16, dtype, 4)
    g = torch.Generator().manual_seed(5)
    slots = torch.randperm(-(-N // ps) * ps + ps, generator=g)[:N].to(torch.int32)
    pages = int(slots.max()) // ps + 1
    kp = torch.zeros((pages, nkv, ps, d), dtype=rt.dtype, device=DEV)
    vp = torch.zeros((pages, nkv, dv, ps), dtype=rt.dtype, device=DEV)
    pos = (torch.arange(N) * 3 + 1).to(torch.int32)
    norms = [torch.rand(d, generator=g) + 0.5 for _ in range(2)] if keys else [None, None]
    ang = PP.rotation_angles(pos, rot, 1000.0, 2.0) if rot else None
    freq = 1000.0 ** (-2.0 * torch.arange(rot // 2, dtype=torch.float64) / rot) / 2.0 if rot else None
    q = torch.empty((N, nh * d), dtype=rt.dtype, device=DEV)
    dev = lambda t: t.to(DEV) if t is not None else None         # noqa: E731
    xd = x.to(DEV).to(rt.dtype)
    K.qk_prepare(xd[:, :row], q, nh, nkv, d, pos.to(DEV), dev(norms[0]), dev(norms[1]), EPS, dev(freq), rot, "neighbours", 1.0,
                 slots.to(DEV), kp, vp, values_are_keys=keys, v_scale=1.25,
                 v_first=None if keys else first.to(DEV).to(rt.dtype)[:, 8:8 + nkv * dv], v_lambda=0.3)
    xd64 = x.double()
    wq, wk = xd64[:, :nh * d].view(N, nh, d), xd64[:, nh * d:(nh + nkv) * d].view(N, nkv, d)
    wv = wk if keys else xd64[:, (nh + nkv) * d:row].view(N, nkv, dv)
    if not keys:
        wv = 0.7 * wv + 0.3 * first.double()[:, 8:8 + nkv * dv].view(N, nkv, dv)
    wv = 1.25 * wv
    if keys:
        wq, wk = PP.unit_rms(wq, EPS) * norms[0].double(), PP.unit_rms(wk, EPS) * norms[1].double()
    if rot:
        wq, wk = PP.rotate_pairs(wq, ang, rot), PP.rotate_pairs(wk, ang, rot)
    assert rel_err(q, wq.reshape(N, -1)) <= PART_TOL[dtype]
    page, off = (slots.long() // ps), (slots.long() % ps)
    assert rel_err(kp.cpu()[page, :, off], wk) <= PART_TOL[dtype]
    assert rel_err(vp.cpu()[page, :, :, off], wv) <= PART_TOL[dtype]


@pytest.mark.parametrize("E,top,groups,keep,renorm,spare", [(8, 3, 4, 2, False, 1), (18, 2, 2, 1, False, 1), (12, 4, 3, 3, True, 0), (5, 1, 5, 2, False, 3),
                                                           (96, 8, 12, 3, False, 1), (130, 5, 2, 1, True, 0), (7, 7, 1, 1, False, 2), (256, 6, 64, 4, False, 0)])
def test_router_with_groups(E, top, groups, keep, renorm, spare):
    """Corrections of both signs (a group whose scores are all below zero can be kept, and its experts chosen), rows that
    hold more than the experts' logits, against the plain choice, where it is no close call."""
    from infernum_amd.kernels import api as K
    g = torch.Generator().manual_seed(E)
    N = 100
    z = torch.randn(N, E + spare, generator=g) * 2
    for shift in (0.0, -3.0):
        corr = torch.randn(E, generator=g) * 0.2 + shift
        s = torch.softmax(z[:, :E].double(), 1)
        ids, wts = PP.choose_experts(s, corr.double(), top, groups, keep)
        sure = PP.choice_margin(s, corr.double(), top, groups, keep) > 1e-5
        got, gw = K.router_softmax_topk(z.to(DEV), corr.to(DEV), top, groups, keep, renorm, E)
        got, gw = got.cpu().long(), gw.cpu().double()
        assert sure.sum() >= 0.8 * N
        for n in range(N):
            if not sure[n]:
                continue
            assert sorted(got[n].tolist()) == sorted(ids[n].tolist())
            want = s[n, got[n]] / (s[n, got[n]].sum() if renorm else 1.0)
            assert torch.allclose(gw[n], want, rtol=1e-5, atol=1e-9)


# ------------------------------------------------------------------------------------ attention kernels on shuffled pages
@pytest.mark.parametrize("nh,nkv,d,dv,ps,window,keep,cap", [
    (6, 2, 32, 32, 16, 20, 3, 7.0), (20, 1, 32, 32, 8, 1, 17, 15.0), (4, 2, 48, 48, 4, 48, 1, 5.0), (4, 4, 16, 16, 12, 33, 40, 0.0),
    (4, 2, 64, 32, 16, 0, 0, 0.0), (2, 1, 16, 48, 16, 0, 0, 0.0), (3, 3, 128, 64, 16, 0, 0, 9.0), (8, 2, 64, 64, 16, 100, 70, 20.0),
    (2, 2, 160, 32, 16, 17, 2, 3.0), (4, 1, 32, 256, 8, 0, 0, 0.0), (5, 1, 80, 16, 16, 64, 64, 0.0)])
def test_matrix_core_attention_against_the_plain_kernel(nh, nkv, d, dv, ps, window, keep, cap):
    """Values of another size, kept first keys, a softcap and sinks, on shuffled pages with NaN wherever no query may
    look: single tokens with the keys in one part and in several, portions that begin anywhere."""
    from infernum_amd.kernels import api as K
    g = torch.Generator().manual_seed(7)
    lens, starts_at = [70, 33, 229, 16, 300, 1], [0, 20, 64, 15, 131, 0]
    B, MB = len(lens), -(-max(lens) // ps)
    num_pages = B * MB + 5
    kp = torch.full((num_pages, nkv, ps, d), float("nan"))
    vp = torch.full((num_pages, nkv, dv, ps), float("nan"))
    perm = torch.randperm(num_pages, generator=g)
    bt = torch.full((B, MB), -1, dtype=torch.int32)
    for b, n in enumerate(lens):
        first = starts_at[b] - window + 1 if window else 0            # the first key that a row of the portions sees
        for pg in range(-(-n // ps)):
            if (pg + 1) * ps > first or pg * ps < keep:
                page = int(perm[b * MB + pg])
                bt[b, pg] = page
                for o in range(ps):
                    t = pg * ps + o
                    if t < n and (t >= first or t < keep):
                        kp[page, :, o] = torch.randn(nkv, d, generator=g)
                        vp[page, :, :, o] = torch.randn(nkv, dv, generator=g)
    dev = lambda t: t.to(torch.bfloat16).to(DEV) if t.dtype.is_floating_point else t.to(DEV)   # noqa: E731
    kp, vp, bt = map(dev, (kp, vp, bt))
    scale = 2.0 / math.sqrt(d)
    for sinks in (None, (torch.randn(nh, generator=g) * 2 + 1).to(DEV)):
        opts = dict(sinks=sinks, keep=keep, softcap=cap)
        q = dev(torch.randn(B, nh * d, generator=g))
        pos = torch.tensor([n - 1 for n in lens], dtype=torch.int32, device=DEV)
        seq = torch.arange(B, dtype=torch.int32, device=DEV)
        wide = torch.full((B, nh * dv + 24), 7.0, dtype=torch.bfloat16, device=DEV)          # columns of wider rows
        want, got = torch.empty((B, nh * dv), dtype=torch.bfloat16, device=DEV), wide[:, 8:8 + nh * dv]
        K.attention_generic(q, kp, vp, want, seq, pos, bt, nh, nkv, d, scale, window, **opts)
        assert torch.isfinite(want.float()).all()
        for splits in (1, 2, 5):
            K.attention_decode(q, kp, vp, got, pos, bt, nh, nkv, d, scale, window, max(lens), num_splits=splits, **opts)
            assert rel_err(got, want.double().cpu()) <= 3e-2, splits
            assert (wide[:, :8] == 7).all() and (wide[:, 8 + nh * dv:] == 7).all()
        news = [n - s0 for n, s0 in zip(lens, starts_at)]
        N = sum(news)
        q = dev(torch.randn(N, nh * d, generator=g))
        starts = torch.tensor([0] + list(torch.tensor(news).cumsum(0)), dtype=torch.int32, device=DEV)
        ctx = torch.tensor(starts_at, dtype=torch.int32, device=DEV)
        seq = torch.cat([torch.full((k,), i, dtype=torch.int32) for i, k in enumerate(news)]).to(DEV)
        pos = torch.cat([torch.arange(f, f + k, dtype=torch.int32) for f, k in zip(starts_at, news)]).to(DEV)
        tiles = torch.tensor([(s_, r) for s_, k in enumerate(news) for r in range(0, k, K.PREFILL_TILE_ROWS)], dtype=torch.int32).to(DEV)
        want, got = (torch.empty((N, nh * dv), dtype=torch.bfloat16, device=DEV) for _ in range(2))
        K.attention_generic(q, kp, vp, want, seq, pos, bt, nh, nkv, d, scale, window, **opts)
        assert torch.isfinite(want.float()).all()
        for shape in (0, 1, 2):
            K.attention_prefill(q, kp, vp, got, starts, ctx, bt, tiles, tiles.shape[0], nh, nkv, d, scale, window, shape,
                                paired=shape == 2, **opts)
            assert rel_err(got, want.double().cpu()) <= 3e-2, shape


@pytest.mark.parametrize("dtype", ["float32"])
@pytest.mark.parametrize("m,T", [(PM.P1["layers"][0]["mixer"]["left"], 60), (PM.P3["layers"][1]["mixer"]["left"], 40)])
def test_plain_attention_kernel_against_the_plain_form(dtype, m, T):
    from infernum_amd.kernels import api as K
    H, G, d, ps = m["heads"], m["kv_heads"], m["dim"], 4
    g = torch.Generator().manual_seed(1)
    q, k, v = torch.randn(T, H, d, generator=g), torch.randn(T, G, d, generator=g), torch.randn(T, G, d + 4, generator=g)
    sinks = torch.randn(H, generator=g)
    kp = k.view(T // ps, ps, G, d).permute(0, 2, 1, 3).contiguous().to(DEV)
    vp = v.view(T // ps, ps, G, d + 4).permute(0, 2, 3, 1).contiguous().to(DEV)
    out = torch.empty((T, H * (d + 4)), device=DEV)
    ar = torch.arange(T, dtype=torch.int32, device=DEV)
    K.attention_generic(q.reshape(T, -1).to(DEV), kp, vp, out, torch.zeros_like(ar), ar, ar[None, :T // ps].contiguous(), H, G, d,
                        0.5, m["mask"]["size"], sinks=sinks.to(DEV), keep=m["mask"]["keep_first"], softcap=m["softcap"])
    want = PP.grouped_attention(q.double(), k.double(), v.double(), 0.5, PP.seen_keys(T, m["mask"]["size"], m["mask"]["keep_first"]),
                                sinks.double(), m["softcap"])
    assert rel_err(out, want) <= 1e-5


# ------------------------------------------------------------------------------------ the mixers alone
ATT_CASES = [(PM.P1["layers"][1]["mixer"], 64, 70), (PM.P2["layers"][1]["mixer"], 100, 45), (PM.P2["layers"][2]["mixer"], 100, 33),
             (PM.P3["layers"][0]["mixer"], 128, 50), (PM.P5["layers"][0]["mixer"], 48, 50), (PM.P5["layers"][2]["mixer"], 48, 90)]
SIDE_CASES = [(PM.P1["layers"][0]["mixer"], 64, 70), (PM.P2["layers"][0]["mixer"], 100, 45), (PM.P3["layers"][1]["mixer"], 128, 50),
              (PM.P3["layers"][4]["mixer"], 128, 90), (PM.P4["layers"][0]["mixer"], 80, 60), (PM.P4["layers"][1]["mixer"], 80, 40)]


@BOTH
@pytest.mark.parametrize("m,W,T", ATT_CASES)
def test_attention_with_one_in_the_denominator_alone(dtype, m, W, T):
    rt = runtime(dtype)
    m = dict(m, v_mix=False)
    mixer, w = _build("softmax_attention", _att_params(m, W), rt, _mixer_weights("attention", m, W, 3))
    x = _x(T, W, dtype, 7)
    want = PP.attention_mixer(x.double(), w, "", m, EPS, {})
    tol = _tol(dtype, want, lambda: PP.attention_mixer(x.double(), w, "", m, EPS, {}, round_to=torch.bfloat16))
    for ps in (4, 16):
        for cuts in CUTS(T):
            got = _run_mixer(mixer, _steps_for(mixer, rt, ps, -(-T // ps) + 2), x, cuts, rt)
            assert rel_err(got.to(rt.dtype), want) <= tol, (ps, cuts[:3])


@BOTH
@pytest.mark.parametrize("m,W,T", SIDE_CASES)
def test_both_mixers_side_by_side_and_each_alone(dtype, m, W, T):
    """The window attention alone (its pages go back while the kept first ones stay), the recurrence alone (slots are
    used again), and both on one product with their factors."""
    rt = runtime(dtype)
    tensors = _mixer_weights("parallel", m, W, 3)
    x = _x(T, W, dtype, 7)
    left = {k[5:]: v for k, v in tensors.items() if k.startswith("left.")}
    right = {k[6:]: v for k, v in tensors.items() if k.startswith("right.")}
    cases = [("softmax_attention", _left_params(m["left"], W), left, lambda w, r: PP.window_attention(x.double(), w, "", m["left"], EPS, r)),
             ("delta_rule", _delta_params(m["right"], W), right, lambda w, r: PP.delta_mixer(x.double(), w, "", m["right"], EPS, r)),
             ("side_by_side", _side_params(m, W), tensors, lambda w, r: PP.parallel_mixer(x.double(), w, "", m, EPS, {}, r))]
    for kind, params, ts, plain in cases:
        mixer, w = _build(kind, params, rt, ts)
        want = plain(w, None)
        tol = _tol(dtype, want, lambda: plain(w, torch.bfloat16))
        if dtype == "float32":          # a head whose sums nearly cancel is divided by a small root mean square
            tol = max(tol, 8.0 * rel_err(plain(w, torch.float32), want))
        for ps in (4, 16):
            steps = _steps_for(mixer, rt, ps, 2 * (-(-T // ps)) + 2, slots=2)
            for i, cuts in enumerate(CUTS(T)):
                got = _run_mixer(mixer, steps, x, cuts, rt, request=f"r{i}")
                mask = m["left"].get("mask")
                if mask and kind != "delta_rule":
                    held = steps.cache.block_table(0, f"r{i}").live_pages()
                    assert len(held) <= -(-mask["size"] // ps) + 1 + -(-mask["keep_first"] // ps)
                steps.cache.release(f"r{i}")
                steps.cache.check()
                assert rel_err(got.to(rt.dtype), want) <= tol, (kind, ps, cuts[:3])


@BOTH
@pytest.mark.parametrize("dim,heads,T", [(16, 2, 40), (30, 3, 33), (64, 2, 21), (96, 1, 19), (128, 2, 17), (130, 1, 9), (256, 1, 9), (1, 2, 20)])
def test_delta_rule_at_many_head_sizes(dtype, dim, heads, T):
    """Against the plain recurrence on the very numbers that enter it: rows of unequal requests in one launch, from
    states that are not zero; then the rest of them token by token."""
    from infernum_amd.kernels import api as K
    rt = runtime(dtype)
    n = heads * dim
    g = torch.Generator().manual_seed(dim)
    lens = [1, T, 8, 2, 75, 16]
    N = sum(lens)
    proj = (torch.randn(N, 3 * n + 5, generator=g) / math.sqrt(dim)).to(rt.dtype)
    w, a = 0.6 + 0.4 * torch.rand(N, n, generator=g), torch.rand(N, n, generator=g)
    slots = torch.tensor([3, 0, 2, 4, 6, 5], dtype=torch.int32)
    state = torch.randn(7, K.delta_state_floats(heads, dim), generator=g)
    S0 = state.view(7, heads, dim, dim).transpose(2, 3)          # kept column by column
    r, k, v = (proj[:, i * n:(i + 1) * n].double().view(N, heads, dim) for i in range(3))
    inv = 1.0 / torch.sqrt((k * k).sum(-1) + 1e-6)
    out = torch.empty((N, n), device=DEV)
    st = state.clone().to(DEV)
    starts = torch.tensor([0] + list(torch.tensor(lens).cumsum(0)), dtype=torch.int32)
    args = [t.to(DEV) for t in (w, a, inv.float())]
    K.delta_scan(proj.to(DEV), 0, n, 2 * n, *args, st, out, starts.to(DEV), slots.to(DEV), heads, dim)
    for i, s in enumerate(slots.tolist()):
        lo, hi = int(starts[i]), int(starts[i + 1])
        for h in range(heads):
            c = slice(h * dim, (h + 1) * dim)
            o, S = PP.delta_recurrence(r[lo:hi, h], k[lo:hi, h], v[lo:hi, h], w[lo:hi, c].double(), a[lo:hi, c].double(), S0[s, h].double())
            assert rel_err(out[lo:hi, c], o) <= 2e-5
            assert rel_err(st.cpu().view(7, heads, dim, dim)[s, h].T, S) <= 2e-5
    assert torch.equal(st[1].cpu(), state[1])                    # a slot that no request holds
    # the same rows token by token: the same bits
    st2, out2 = state.clone().to(DEV), torch.empty_like(out)
    done = [0] * len(lens)
    while any(d < L for d, L in zip(done, lens)):
        live = [i for i in range(len(lens)) if done[i] < lens[i]]
        rows = torch.tensor([int(starts[i]) + done[i] for i in live])
        y = torch.empty((len(live), n), device=DEV)
        K.delta_scan(proj[rows].contiguous().to(DEV), 0, n, 2 * n, *[t[rows.to(DEV)].contiguous() for t in args], st2, y,
                     torch.arange(len(live) + 1, dtype=torch.int32, device=DEV), slots[live].to(DEV), heads, dim)
        out2[rows.to(DEV)] = y
        for i in live:
            done[i] += 1
    assert torch.equal(out, out2) and torch.equal(st, st2)
    # the same rows in chunks, but for the first request's, whose tokens a step brings alone
    st3, out3 = state.clone().to(DEV), torch.full_like(out, float("nan"))
    tiles = torch.tensor([(i, r) for i, L in list(enumerate(lens))[1:] for r in range(0, L, K.PREFILL_TILE_ROWS)][::-1], dtype=torch.int32)
    K.delta_chunked(proj.to(DEV), 0, n, 2 * n, *args, st3, out3, starts.to(DEV), slots.to(DEV), tiles.to(DEV), tiles.shape[0], 1,
                    len(lens) - 1, heads, dim)
    lo = lens[0]
    assert rel_err(out3[lo:], out[lo:].double().cpu()) <= 2e-5
    assert rel_err(st3, torch.where(torch.arange(7)[:, None] == slots[0], state, st.cpu()).double()) <= 2e-5


@BOTH
def test_a_state_that_reaches_hundreds_of_tokens_back(dtype):
    """A head that hardly decays and takes nothing out carries what token 3 wrote over 600 tokens, whole and decoded."""
    m, W, T = {"heads": 2, "dim": 16}, 32, 640
    rt = runtime(dtype)
    p = {"left": PM._left(1, 1, 16, 1.0), "right": m, "left_scale": 1.0, "right_scale": 1.0}
    w = _mixer_weights("parallel", p, W, 5, "mix.right.")
    w["w0"][:16], w["w1"] = -11.0, w["w1"] * 0.02
    w["a"][:16], w["a.b"][:16] = 0.0, -20.0
    w["a.b"][16:] = 2.0                                     # the second head forgets
    w["k"][:, 1:] = w["v"][:, 1:] = 0.0                     # only a token whose first place is not zero writes
    w["r"] = 0.05 * w["r"]                                  # and every token reads along what was written
    w["r"][:, 1] = 2.0 * w["k"][:, 0]
    x = _x(T, W, dtype, 11)
    x[:, 0], x[:, 1] = 0.0, 1.0
    x[3, 0] = 6.0
    mixer, w = _build("delta_rule", _delta_params(m, W), rt, w)
    want = PP.delta_mixer(x.double(), w, "", m, EPS)
    other = x.clone()
    other[3, 0] = 0.0
    without = PP.delta_mixer(other.double(), w, "", m, EPS)
    tol = _tol(dtype, want, lambda: PP.delta_mixer(x.double(), w, "", m, EPS, torch.bfloat16))
    assert (want[-1] - without[-1]).abs().max() > 10 * tol * want.pow(2).mean().sqrt()
    for cuts in ([T], [300, 209, 1, 1, 1, 1, 1, T - 514], [3, 1, T - 10] + [1] * 6):
        got = _run_mixer(mixer, _steps_for(mixer, rt, 16, 4, slots=2), x, cuts, rt)
        assert rel_err(got.to(rt.dtype), want) <= tol, cuts[:2]


def _standing_out(dtype, T, star, size, keep, d=16):
    """One head whose queries all point one way; the star's key alone points that way, the others' lie across it.
    Values are the keys before their norm: the star's is 5 along the first place, and the output projection passes that
    place on, so that a row shows about 5 where it sees the star and nothing where it does not."""
    W = 8
    rt = runtime(dtype)
    m = {"heads": 1, "kv_heads": 1, "dim": d, "vdim": d, "scale": 1.0, "softcap": 50.0, "mask": {"size": size, "keep_first": keep}}
    z = lambda *s: torch.zeros(s, dtype=torch.float64)          # noqa: E731
    w = {"q": z(d, W), "k": z(d, W), "o": z(W, d), "q.norm": torch.ones(d), "k.norm": torch.ones(d), "sink": torch.tensor([-3.0])}
    w["q"][0, 0] = 1.0
    w["k"][0, 1], w["k"][1, 2] = 5.0, 1.0
    w["o"][0, 0] = 1.0
    x = torch.zeros(T, W)
    x[:, 0], x[:, 2] = 1.0, 1.0
    x[star, 1], x[star, 2] = 1.0, 0.0
    mixer, w = _build("softmax_attention", _left_params(m, W), rt, w)
    return rt, mixer, w, m, x


@BOTH
@pytest.mark.parametrize("star,size,keep", [(9, 7, 4), (3, 7, 4), (4, 7, 4), (16, 5, 17), (17, 5, 17), (0, 1, 1), (1, 1, 1), (15, 16, 0), (31, 3, 31),
                                            (30, 3, 31)])
def test_a_key_that_stands_out_at_the_windows_edge_and_among_the_first(dtype, star, size, keep):
    """Rows star .. star + size - 1 see the star; later rows only when it is one of the kept first positions.  Whole,
    decoded across the edge, in portions that begin at the edge, in pairs; pages of 4 and 16."""
    T = 80
    rt, mixer, w, m, x = _standing_out(dtype, T, star, size, keep)
    want = PP.window_attention(x.double(), w, "", m, EPS)
    last_in = star + size - 1
    shows = want[:, 0]
    assert (shows[:star].abs() < 0.1).all()
    assert (shows[star:last_in + 1] > 4.5).all()
    assert (shows[last_in + 1:] > 4.5).all() if star < keep else (shows[last_in + 1:].abs() < 0.1).all()
    tol = _tol(dtype, want, lambda: PP.window_attention(x.double(), w, "", m, EPS, torch.bfloat16))
    edge = last_in + 1
    for ps in (4, 16):
        for cuts in CUTS(T) + [[edge, T - edge], [edge - 1] * (edge > 1) + [1] * 5 + [T - edge - 5 + (edge == 1)],
                               [edge] + [1] * (T - edge)]:
            cuts = [c for c in cuts if c > 0]
            cuts[-1] += T - sum(cuts)
            got = _run_mixer(mixer, _steps_for(mixer, rt, ps, T // ps + 2), x, cuts, rt)
            assert rel_err(got.to(rt.dtype), want) <= tol, (ps, cuts[:3])


@BOTH
def test_a_key_far_back_among_hundreds(dtype):
    """The key of position 2 alone answers the query 500 positions later: through the kept first positions of a window
    of 9, and in attention over all keys; whole, decoded and in portions."""
    T, star = 520, 2
    rt, mixer, w, m, x = _standing_out(dtype, T, star, 9, 3)
    want = PP.window_attention(x.double(), w, "", m, EPS)
    assert (want[star:, 0] > 4.5).all()
    tol = _tol(dtype, want, lambda: PP.window_attention(x.double(), w, "", m, EPS, torch.bfloat16))
    for cuts in ([T], [T - 20] + [1] * 20, [63, 2, 100, 64, 1, 2, T - 232]):
        got = _run_mixer(mixer, _steps_for(mixer, rt, 16, T // 16 + 2), x, cuts, rt)
        assert rel_err(got.to(rt.dtype), want) <= tol, cuts[:2]
    full = {"heads": 1, "kv_heads": 1, "dim": 16, "vdim": 32, "scale": 12.0}
    W = 8
    z = lambda *s: torch.zeros(s, dtype=torch.float64)          # noqa: E731
    w = {"q": z(16, W), "k": z(16, W), "v": z(32, W), "o": z(W, 32)}
    w["q"][0, 0] = w["k"][0, 1] = w["k"][1, 2] = 1.0
    w["v"][0, 1], w["o"][0, 0] = 5.0, 1.0
    mixer, w = _build("softmax_attention", _att_params(full, W), rt, w)
    want = PP.attention_mixer(x.double(), w, "", full, EPS, {})
    assert (want[star:, 0] > 4.5).all()
    for cuts in ([T], [T - 20] + [1] * 20, [63, 2, 100, 64, 1, 2, T - 232]):
        got = _run_mixer(mixer, _steps_for(mixer, rt, 16, T // 16 + 2), x, cuts, rt)
        assert rel_err(got.to(rt.dtype), want) <= PART_TOL[dtype], cuts[:2]


@BOTH
def test_values_mixed_with_an_earlier_layers(dtype):
    """Two attention mixers in a row on inputs of their own: the second's values are mixed with the first's, and the
    mixture is what its pages hold for later steps."""
    rt = runtime(dtype)
    W, T = 64, 50
    m1, m2 = PM.P1["layers"][1]["mixer"], PM.P1["layers"][4]["mixer"]
    t2 = _mixer_weights("attention", m2, W, 4)
    t2["vmix"] = torch.tensor(0.625)
    a, wa = _build("softmax_attention", _att_params(m1, W, "first"), rt, _mixer_weights("attention", m1, W, 3))
    b, wb = _build("softmax_attention", _att_params(m2, W, "mixed"), rt, t2)
    x, y = _x(T, W, dtype, 5), _x(T, W, dtype, 6)
    shared = {}
    PP.attention_mixer(x.double(), wa, "", m1, EPS, shared)
    want = PP.attention_mixer(y.double(), wb, "", m2, EPS, shared)
    alone = PP.attention_mixer(y.double(), wb, "", dict(m2, v_mix=False), EPS, {})
    assert rel_err(alone, want) > 0.1
    sr = {}
    PP.attention_mixer(x.double(), wa, "", m1, EPS, sr, torch.bfloat16)
    tol = _tol(dtype, want, lambda: PP.attention_mixer(y.double(), wb, "", m2, EPS, sr, torch.bfloat16))
    for cuts in CUTS(T):
        steps = Steps([(a.cache_spec(), None), (b.cache_spec(), None)], rt, page_size=8, num_pages=20, poison=True)
        out, p = [], 0
        for n in cuts:
            ctx, packed = steps.begin([("a", n)])
            a.forward(x[p:p + n].to(DEV).to(rt.dtype), ctx, steps.views[0])
            out.append(dense(b.forward(y[p:p + n].to(DEV).to(rt.dtype), ctx, steps.views[1]), rt).float().cpu())
            steps.end(packed)
            p += n
        assert rel_err(torch.cat(out).to(rt.dtype), want) <= tol, cuts[:3]


@BOTH
@pytest.mark.parametrize("mlp,W,N", [(PM.P1["layers"][0]["mlp"], 64, 60), (PM.P2["layers"][0]["mlp"], 100, 9), (PM.P2["layers"][2]["mlp"], 100, 40),
                                     (PM.P3["layers"][1]["mlp"], 128, 1), (PM.P3["layers"][2]["mlp"], 128, 70), (PM.P5["layers"][1]["mlp"], 48, 30),
                                     (PM._moe(64, 4, 2, 4, (2, 1), 64), 64, 300), (PM._moe(64, 6, 3, 3, (3, 2)), 128, 200)])
def test_routed_experts_alone(dtype, mlp, W, N):
    """Groups, a correction, identity experts and the gated shared expert; by natural routers (where no choice is a
    close call) and by corrections that decide alone; few tokens and so many that the grouped product takes them."""
    from infernum_amd.parts import PartSpec, make_part
    from infernum_amd.config.pamazen import MoeConfig
    from infernum_amd.config.base import KeyReader
    rt = runtime(dtype)
    f = MoeConfig.from_reader(KeyReader(mlp))
    mixer = PM._attn(1, 1, 16, 16, 1.0)
    ts = {k[4:]: v for k, v in _layer_weights({"type": "attention", "mixer": mixer, "mlp": mlp}, W, 8).items() if k.startswith("mlp.")}
    x = _x(N, W, dtype, 9)
    for how in ("natural", "decided"):
        if how == "decided":
            ts["correction"] = PM.decided({}, {"mlp.correction": ts["correction"]}, 3)["mlp.correction"].double()
        part = make_part("feed_forward", PartSpec("routed_experts", {
            "hidden_size": W, "intermediate_size": f.ff, "num_experts": f.experts, "top": f.top, "gated": True, "limit": None,
            "alpha": 1.0, "up_shift": 0.0, "router": "softmax_top", "renorm": False, "groups": f.groups, "keep_groups": f.keep,
            "identity": f.identity, "shared_ff": f.shared_ff, "shared_gate": "shared.sg" if f.shared_ff else None}), rt)
        part.load({n: ts[n].float().to(DEV).to(rt.dtype if ws.follows_compute_dtype or rt.is_fp32 else torch.float32)
                   for n, ws in part.weights().items()})
        margins = []
        want = PP.routed_experts(x.double(), ts, "", mlp, margins=margins)
        sure = margins[0] > 3e-4
        assert sure.sum() >= 0.7 * N
        rounded = PP.routed_experts(x.double(), ts, "", mlp, torch.bfloat16)
        got = dense(part.forward(x.to(DEV).to(rt.dtype)), rt).cpu()
        assert torch.isfinite(got.float()).all()
        assert rel_err(got[sure], want[sure]) <= _tol(dtype, want[sure], lambda: rounded[sure])


@BOTH
def test_requests_of_unequal_length_side_by_side_and_alone(dtype):
    """A batch of unequal requests in steps of unequal portions: every row as if its request were alone."""
    m, W = PM.P1["layers"][0]["mixer"], 64
    rt = runtime(dtype)
    mixer, w = _build("side_by_side", _side_params(m, W), rt, _mixer_weights("parallel", m, W, 4))
    lens = {"a": 1, "b": 130, "c": 64, "d": 65, "e": 1, "f": 7}
    xs = {r: _x(n + 3, W, dtype, 20 + i) for i, (r, n) in enumerate(lens.items())}
    want = {r: PP.parallel_mixer(x.double(), w, "", m, EPS, {}) for r, x in xs.items()}
    steps = _steps_for(mixer, rt, 16, 40, slots=6)
    got = {r: [] for r in lens}
    for portion in (lambda r: lens[r], lambda r: 1, lambda r: 2):
        done = {r: sum(t.shape[0] for t in got[r]) for r in lens}
        ctx, packed = steps.begin([(r, portion(r)) for r in lens])
        rows = torch.cat([xs[e.request][done[e.request]:done[e.request] + len(e.tokens)] for e in packed.batch])
        y = dense(mixer.forward(rows.to(DEV).to(rt.dtype), ctx, steps.views[0]), rt).float().cpu()
        steps.end(packed)
        at = 0
        for e in packed.batch:
            got[e.request].append(y[at:at + len(e.tokens)])
            at += len(e.tokens)
    for r in lens:
        tol = _tol(dtype, want[r], lambda: PP.parallel_mixer(xs[r].double(), w, "", m, EPS, {}, torch.bfloat16))
        assert rel_err(torch.cat(got[r]).to(rt.dtype), want[r]) <= tol, r


# ------------------------------------------------------------------------------------ the engine
TOLERANCE = {}


def _requests(cfg, w, lengths, seed, margins=None):
    reqs = TT.make_requests(cfg["vocab"], lengths, seed=seed)
    return reqs, {r: PP.forward(cfg, w, t, margins=margins) for r, t in reqs.items()}


class _Model:
    """A model folder per compute type.  In 32-bit the routers choose by themselves (no choice of the requests is
    closer than rounding can turn); in bfloat16 the corrections decide alone."""

    def __init__(self, name, root):
        self.name, self.cfg = name, PM.RAW[name]
        natural = PP.random_weights(self.cfg, PM.SEED[name])
        self.w = {"float32": natural, "bfloat16": PM.decided(self.cfg, natural)}
        self.dir, self.reqs, self.ref, self.mreqs, self.mref = {}, None, {}, None, {}
        for dtype, w in self.w.items():
            self.dir[dtype] = str(root / dtype)
            PM.write_model(self.cfg, self.dir[dtype], weights=w)
            margins = []
            self.reqs, self.ref[dtype] = _requests(self.cfg, w, LENGTHS[name], 11, margins)
            self.mreqs, self.mref[dtype] = _requests(self.cfg, w, MIXED[name], 23, margins)
            assert min(float(m.min()) for m in margins) > 1e-5
            to = torch.bfloat16 if dtype == "bfloat16" else torch.float32
            cost = 0.0
            for group, refs in ((self.reqs, self.ref[dtype]), (self.mreqs, self.mref[dtype])):
                for r, t in group.items():
                    cost = max(cost, (PP.forward(self.cfg, w, t, round_to=to) - refs[r]).abs().max().item() / refs[r].pow(2).mean().sqrt().item())
            # in 32-bit the plain model rounds what is stored between kernels and none of the sums inside them
            TOLERANCE[name, dtype] = max(TOL[dtype], (3.0 if dtype == "bfloat16" else 8.0) * cost)


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    return {name: _Model(name, tmp_path_factory.mktemp(name)) for name in NAMES}


def _engine(model_dir, dtype, page_size, num_pages, slots=8, **kw):
    from infernum_amd import CacheConfig, Engine
    return Engine.from_pretrained(model_dir, dtype=dtype, **kw,
                                  cache_config=CacheConfig(page_size=page_size, num_pages=num_pages,
                                                           num_state_slots=slots, poison_freed_pages=True))


def _check(got, ref, dtype, what, name):
    assert all(torch.isfinite(t).all() for t in got.values())
    worst, rms, where = TT.error_against(got, ref)
    print(f"{what}: max|diff| = {worst:.3e}, rms of logits = {rms:.3e}, ratio {worst / rms:.2e} at {where} over {len(got)} places")
    assert worst <= TOLERANCE[name, dtype] * rms, f"{what}: max|diff| {worst:.3e} > {TOLERANCE[name, dtype]} * rms {rms:.3e} at {where}"


@BOTH
@pytest.mark.parametrize("name", NAMES)
def test_the_stream_after_every_layer(models, tmp_path, name, dtype):
    """The logits of the models made of the first k layers (the same tensors), k = 1, 2, ...: a layer that differs
    shows at its own k.  The parts' own way gives what the step's program gives."""
    import copy
    from infernum_amd.engine import StepEntry
    m = models[name]
    toks = m.reqs["r2"]
    for k in range(1, len(m.cfg["layers"]) + 1):
        sub = copy.deepcopy(m.cfg)
        sub["layers"] = sub["layers"][:k]
        keep = {n: t for n, t in m.w[dtype].items() if not (n[0] == "l" and n[1].isdigit()) or int(n[1:n.index(".")]) < k}
        sd = str(tmp_path / f"first{k}")
        PM.write_model(sub, sd, weights=keep)
        logits = _engine(sd, dtype, PAGE[name], 64).step([StepEntry("a", toks, list(range(len(toks))))]).cpu()
        _check({("a", p): logits[p] for p in range(len(toks))}, {"a": PP.forward(sub, keep, toks)}, dtype,
               f"{name} {dtype} first {k} layers", name)
        parts = _engine(sd, dtype, PAGE[name], 64, executor="parts").step([StepEntry("a", toks, list(range(len(toks))))]).cpu()
        assert torch.equal(parts, logits)


@BOTH
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("how", ["whole", "tail", "portions", "one_by_one"])
def test_one_request_at_a_time(models, name, dtype, how):
    m = models[name]
    eng = _engine(m.dir[dtype], dtype, PAGE[name], 64)
    steps = {"whole": TT.trace_whole, "tail": lambda r: TT.trace_tail_one_by_one(r, 40), "portions": TT.trace_portions,
             "one_by_one": lambda r: TT.trace_tail_one_by_one(r, 10 ** 6)}[how](m.reqs)
    _check(TT.run_steps(eng, steps), m.ref[dtype], dtype, f"{name} {dtype} {how}", name)
    eng.cache.check()
    assert all(eng.cache.free_pages(g) == 64 for g in range(len(eng.cache.groups)))
    if eng.program is not None:
        eng.program.check_guards()
        assert eng.program.num_python_ops == 0             # every part wrote its own launches


@BOTH
@pytest.mark.parametrize("name", NAMES)
def test_mixed_batches_with_pages_and_slots_used_again(models, name, dtype):
    m = models[name]
    prompt_len = {r: max(2, len(t) - 20 - 7 * i) for i, (r, t) in enumerate(m.mreqs.items())}
    steps, max_tokens = TT.trace_mixed(m.mreqs, prompt_len, seed=5)
    ps = PAGE[name]
    eng = _engine(m.dir[dtype], dtype, ps, -(-max_tokens // ps), slots=4)      # four slots for up to four live of more requests
    assert sum(-(-len(t) // 64) * 64 for t in m.mreqs.values()) > max_tokens   # the pool cannot hold them all: pages come back
    assert len(m.mreqs) > 4
    got = TT.run_steps(eng, steps)
    _check(got, m.mref[dtype], dtype, f"{name} {dtype} mixed", name)
    eng.cache.check()
    if dtype == "float32":          # the same rows from a batch and alone
        alone = TT.run_steps(_engine(m.dir[dtype], dtype, ps, 64), TT.trace_whole(m.mreqs))
        assert all(rel_err(got[k], alone[k].cpu()) <= 1e-5 for k in got)


@BOTH
@pytest.mark.parametrize("name", ["P1", "P3", "P4"])
def test_long_decoding(models, name, dtype):
    """A short prompt, then 150 tokens one by one: the state moves on 150 times, the windows pass over decoded tokens,
    pages fill, begin and go back; decode steps are replayed from graphs after the first two."""
    m = models[name]
    w = m.w[dtype]
    reqs, ref = _requests(m.cfg, w, (160,), 3)
    cost = max((PP.forward(m.cfg, w, t, round_to=torch.float32 if dtype == "float32" else torch.bfloat16) - ref[r]).abs().max().item()
               / ref[r].pow(2).mean().sqrt().item() for r, t in reqs.items())
    TOLERANCE[name, dtype] = max(TOLERANCE[name, dtype], (8.0 if dtype == "float32" else 3.0) * cost)
    eng = _engine(m.dir[dtype], dtype, 16, 12)
    _check(TT.run_steps(eng, TT.trace_tail_one_by_one(reqs, 150)), ref, dtype, f"{name} {dtype} long decoding", name)
    assert eng.graph_replays > 100


def test_greedy_generation_through_the_scheduler(models):
    """Runtime.generate_batch (scheduler, portions, the sampler's argmax) against the plain model's greedy tokens,
    in 32-bit; prompts of unequal length, more requests than run at once."""
    from infernum_amd import BatchConfig, GenerateOptions, Runtime
    m = models["P1"]
    prompts = list(TT.make_requests(m.cfg["vocab"], (5, 31, 2, 18, 9), seed=9).values())
    rt = Runtime.from_pretrained(m.dir["float32"], dtype="float32",
                                 batch_config=BatchConfig(block_size=16, num_blocks=24, max_batch_size=3, max_prefill_tokens=8,
                                                          max_tokens_per_step=16, step_token_multiple=1))
    outs = rt.generate_batch(prompts, GenerateOptions(max_new_tokens=12))
    for p, got in zip(prompts, outs):
        toks = list(p)
        for _ in range(12):
            toks.append(int(PP.forward(m.cfg, m.w["float32"], toks)[-1].argmax()))
        assert list(got) == toks[len(p):], (p, got, toks[len(p):])


@BOTH
def test_trace_run_and_generate_programs(models, tmp_path, dtype):
    """bin/trace_run and bin/generate as a user starts them: the model class comes from config.json; steps on standard
    input, logits in files; generated tokens on standard output."""
    import json
    import os
    import subprocess
    import sys
    import numpy as np
    m = models["P3"]
    reqs = m.mreqs
    prompt_len = {r: max(2, len(t) - 12) for r, t in reqs.items()}
    steps, max_tokens = TT.trace_mixed(reqs, prompt_len, seed=4)
    out = tmp_path / "out"
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", m.dir[dtype], "--dtype", dtype,
                           "--out", str(out), "--max-tokens", str(max_tokens)],
                          input="".join(json.dumps(s) + "\n" for s in steps), text=True, capture_output=True, timeout=100)
    assert proc.returncode == 0, proc.stderr[-3000:]
    assert proc.stdout.split("\n")[:-1] == [f"done {s['step']}" for s in steps]
    pos, got = {}, {}
    for s in steps:
        n_want = sum(len(e["want"]) for e in s["entries"])
        arr = np.fromfile(out / f"{s['step']}.f32", dtype="<f4").reshape(n_want, m.cfg["vocab"])
        row = 0
        for e in s["entries"]:
            base = pos.get(e["id"], 0)
            for k in e["want"]:
                got[(e["id"], base + k)] = torch.from_numpy(arr[row].copy())
                row += 1
            pos[e["id"]] = base + len(e["tokens"])
    _check(got, m.mref[dtype], dtype, f"trace_run P3 {dtype} mixed", "P3")
    if dtype == "float32":
        prompt = reqs["r4"][:9]
        gen = subprocess.run([sys.executable, os.path.join(root, "bin", "generate"), "-m", m.dir[dtype], "--prompt-ids",
                              ",".join(map(str, prompt)), "-n", "6", "--greedy", "--dtype", "float32"],
                             text=True, capture_output=True, timeout=100)
        assert gen.returncode == 0, gen.stderr[-3000:]
        toks = list(prompt)
        for _ in range(6):
            toks.append(int(PP.forward(m.cfg, m.w[dtype], toks)[-1].argmax()))
        assert " " + " ".join(map(str, toks[9:])) + "\n" in gen.stdout, gen.stdout[-2000:]
