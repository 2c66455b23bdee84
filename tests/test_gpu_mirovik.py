"""The Mirovik decoder on the GPU against the plain implementation (plain_mirovik.py): each mechanism alone, then the
engine on small models of other sizes than any real one: whole prompts, the tail decoded token by token, portions down to
two tokens, mixed batches over pools so small that pages and state slots are used again (freed pages hold NaN), keys at every
edge of the bias by distance, far back among hundreds, states that reach hundreds of tokens back, long decoding from graphs,
and greedy generation through the runtime and its scheduler."""
import math

import pytest
import torch

import mirovik_models as MM
import plain_mirovik as MP
import trace_tools as TT
from part_harness import DEV, TOL as PART_TOL, Steps, dense, rel_err, runtime

pytestmark = pytest.mark.gpu
BOTH = pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
# largest |difference| of a logit as a fraction of the RMS of the plain logits
TOL = {"float32": 3e-5, "bfloat16": 6e-2}
NAMES = ["V1", "V2", "V3", "V4", "V5"]
LENGTHS = {"V1": (1, 7, 45, 83, 130), "V2": (3, 61, 33, 97), "V3": (9, 70, 121), "V4": (2, 17, 64, 150), "V5": (1, 64, 65, 140)}
MIXED = {"V1": (70, 131, 64, 150, 33, 97, 66, 81), "V2": (150, 165, 120, 190, 147), "V3": (129, 65, 90, 47, 72, 99),
         "V4": (70, 131, 64, 150, 33, 97), "V5": (150, 100, 64, 190, 129, 77)}
PAGE = {"V1": 16, "V2": 4, "V3": 8, "V4": 16, "V5": 12}
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


def _layer_weights(layer, W, seed):
    w = MP.random_weights({"vocab": 4, "width": W, "layers": [layer]}, seed)
    return {k[3:]: v.double() for k, v in w.items() if k.startswith("l0.")}


def _mixer_weights(kind, m, W, seed):
    return {k[4:]: v for k, v in _layer_weights({"type": kind, "mixer": m, "mlp": None}, W, seed).items() if k.startswith("mix.")}


def _left_params(m, W):
    return {"hidden_size": W, "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "head_dim": m["dim"],
            "value_dim": m["vdim"], "scale": m["scale"], "qk_norm": "rows", "norm_eps": EPS,
            "distance_bias": {"far": m["bias_max"], "rows": m["buckets"]}, "output_gate": True}


def _right_params(m, W):
    rot = m.get("rot")
    position = {"kind": "rope", "params": {"head_dim": m["dim"], "theta": rot["base"], "rotary_dim": rot["dims"]}} if rot else None
    return {"hidden_size": W, "num_heads": m["heads"], "head_dim": m["dim"], "value_dim": m["vdim"], "decay": m["decay"],
            "norm_eps": EPS, "position": position}


def _side_params(m, W):
    return {"hidden_size": W, "mixers": {
        "left": {"kind": "softmax_attention", "scale": m["left_scale"], "params": _left_params(m["left"], W)},
        "right": {"kind": "retention", "scale": m["right_scale"], "params": _right_params(m["right"], W)}}}


def _mamba_params(m, W):
    return {"hidden_size": W, "inner": m["inner"], "state_size": m["state"], "dt_rank": m["dt_rank"], "conv_taps": m["conv"]}


def _build(kind, params, rt, tensors, category="mixer"):
    from infernum_amd.parts import PartSpec, make_part
    part = make_part(category, PartSpec(kind, params), rt)
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
@pytest.mark.parametrize("nh,nkv,d,dv,ps,N", [(4, 2, 32, 16, 16, 37), (3, 3, 12, 10, 4, 9), (20, 1, 16, 48, 8, 40), (2, 1, 64, 128, 12, 130),
                                             (5, 5, 20, 20, 4, 7), (1, 1, 8, 8, 4, 1), (32, 4, 128, 64, 16, 21)])
def test_rows_into_queries_keys_and_values_normed_over_all_heads(dtype, nh, nkv, d, dv, ps, N):
    from infernum_amd.kernels import api as K
    rt = runtime(dtype)
    row = (nh + nkv) * d + nkv * dv
    x = _x(N, row + 8, dtype, 3)
    g = torch.Generator().manual_seed(5)
    slots = torch.randperm(-(-N // ps) * ps + ps, generator=g)[:N].to(torch.int32)
    if N > 5:
        slots[4] = -1                                        # a token without a place writes nowhere
    pages = int(slots.max()) // ps + 1
    kp = torch.zeros((pages, nkv, ps, d), dtype=rt.dtype, device=DEV)
    vp = torch.zeros((pages, nkv, dv, ps), dtype=rt.dtype, device=DEV)
    wq, wk = torch.rand(nh * d, generator=g) + 0.5, torch.rand(nkv * d, generator=g) + 0.5
    q = torch.empty((N, nh * d), dtype=rt.dtype, device=DEV)
    K.qk_rows_prepare(x.to(DEV).to(rt.dtype)[:, :row], q, nh, nkv, d, wq.to(DEV), wk.to(DEV), EPS, slots.to(DEV), kp, vp, 1.25)
    xd = x.double()
    nq, nk = nh * d, nkv * d
    want_q = MP.unit_rms(xd[:, :nq], EPS) * wq.double()
    want_k = (MP.unit_rms(xd[:, nq:nq + nk], EPS) * wk.double()).view(N, nkv, d)
    want_v = 1.25 * xd[:, nq + nk:row].view(N, nkv, dv)
    assert rel_err(q, want_q) <= PART_TOL[dtype]
    has = slots >= 0
    page, off = (slots.long() // ps)[has], (slots.long() % ps)[has]
    assert rel_err(kp.cpu()[page, :, off], want_k[has]) <= PART_TOL[dtype]
    assert rel_err(vp.cpu()[page, :, :, off], want_v[has]) <= PART_TOL[dtype]
    assert int((kp.abs().sum(dim=(1, 3)) > 0).sum()) == int(has.sum())


@pytest.mark.parametrize("N,H,code", [(1, 64, torch.float32), (37, 100, torch.bfloat16), (3, 2051, torch.bfloat16)])
def test_a_vector_added_to_every_row(N, H, code):
    from infernum_amd.kernels import api as K
    g = torch.Generator().manual_seed(N)
    h, v = torch.randn(N, H, generator=g), torch.randn(H, generator=g).to(code)
    got = K.add_vector(h.clone().to(DEV), v.to(DEV)).cpu()
    assert torch.equal(got, h + v.float())


@pytest.mark.parametrize("E,top,spare,scale", [(8, 1, 0, 2.0), (6, 6, 1, 1.0), (130, 5, 0, 3.0), (300, 4, 2, 2.0), (1, 1, 0, 1.0), (16, 3, 0, 40.0)])
def test_router_with_sigmoid_scores(E, top, spare, scale):
    """The last case has logits whose sigmoids are equal in fp32: the choice still goes by the larger logit."""
    from infernum_amd.kernels import api as K
    g = torch.Generator().manual_seed(E)
    z = torch.randn(50, E + spare, generator=g) * scale
    ids, wts = K.router_softmax_topk(z.to(DEV), None, top, 1, 1, False, E, sigmoid=True)
    want = z[:, :E].topk(top, dim=1)
    assert torch.equal(ids.cpu().long(), want.indices)
    assert torch.allclose(wts.cpu().double(), MP.sigmoid(want.values.double()), rtol=1e-6, atol=1e-12)
    corr = torch.randn(E, generator=g) * 0.3
    s = MP.sigmoid(z[:, :E].double())
    order = (s + corr.double()).sort(dim=1, descending=True).values
    sure = (order[:, top - 1] - order[:, top] > 1e-5) if top < E else torch.ones(50, dtype=torch.bool)
    ids, wts = K.router_softmax_topk(z.to(DEV), corr.to(DEV), top, 1, 1, True, E, sigmoid=True)
    want = (s + corr.double()).topk(top, dim=1).indices
    for n in range(50):
        if sure[n]:
            got = ids[n].cpu().long()
            assert sorted(got.tolist()) == sorted(want[n].tolist())
            assert torch.allclose(wts[n].cpu().double(), s[n, got] / s[n, got].sum(), rtol=1e-5, atol=1e-9)


# ------------------------------------------------------------------------------------ attention kernels on shuffled pages
@pytest.mark.parametrize("nh,nkv,d,dv,ps,rows,far,gate,window,cap", [
    (4, 2, 32, 16, 16, 20, 40.0, True, 0, 0.0), (20, 1, 16, 16, 8, 64, 300.0, True, 0, 0.0), (3, 3, 48, 80, 12, 2, 3.0, True, 0, 0.0),
    (2, 1, 64, 64, 16, 16, 33.0, False, 0, 0.0), (4, 2, 80, 48, 4, 32, 128.0, True, 0, 0.0), (6, 2, 128, 128, 16, 14, 30.0, True, 20, 0.0),
    (2, 2, 160, 32, 16, 8, 70.0, True, 0, 0.0), (4, 4, 16, 32, 16, 32, 2000.0, True, 33, 9.0), (8, 1, 64, 64, 16, 0, 0.0, True, 0, 0.0)])
def test_matrix_core_attention_against_the_plain_kernel(nh, nkv, d, dv, ps, rows, far, gate, window, cap):
    """A bias by distance and gates, on shuffled pages with NaN wherever no query may look: single tokens with the keys in
    one part and in several, portions that begin anywhere; with a window and a softcap beside them as well."""
    from infernum_amd.kernels import api as K
    from infernum_amd.parts.softmax_attention import bias_by_distance
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
            if (pg + 1) * ps > first:
                page = int(perm[b * MB + pg])
                bt[b, pg] = page
                for o in range(ps):
                    t = pg * ps + o
                    if t < n and t >= first:
                        kp[page, :, o] = torch.randn(nkv, d, generator=g)
                        vp[page, :, :, o] = torch.randn(nkv, dv, generator=g)
    dev = lambda t: t.to(torch.bfloat16).to(DEV) if t.dtype.is_floating_point else t.to(DEV)   # noqa: E731
    kp, vp, bt = map(dev, (kp, vp, bt))
    scale = 1.0 / math.sqrt(d)
    bias = K.distance_table(bias_by_distance(3.0 * torch.randn(rows, nh, generator=g), far)).to(DEV) if rows else None

    def gates(n):                                                     # columns of wider rows
        return dev(torch.randn(n, nh * dv + 16, generator=g))[:, 8:8 + nh * dv] if gate else None

    q = dev(torch.randn(B, nh * d, generator=g))
    pos = torch.tensor([n - 1 for n in lens], dtype=torch.int32, device=DEV)
    seq = torch.arange(B, dtype=torch.int32, device=DEV)
    wide = torch.full((B, nh * dv + 24), 7.0, dtype=torch.bfloat16, device=DEV)
    want, got = torch.empty((B, nh * dv), dtype=torch.bfloat16, device=DEV), wide[:, 8:8 + nh * dv]
    opts = dict(softcap=cap, bias=bias, gate=gates(B))
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
    opts["gate"] = gates(N)
    K.attention_generic(q, kp, vp, want, seq, pos, bt, nh, nkv, d, scale, window, **opts)
    assert torch.isfinite(want.float()).all()
    for shape in (0, 1, 2):
        K.attention_prefill(q, kp, vp, got, starts, ctx, bt, tiles, tiles.shape[0], nh, nkv, d, scale, window, shape,
                            paired=shape == 2, **opts)
        assert rel_err(got, want.double().cpu()) <= 3e-2, shape


def test_plain_attention_kernel_against_the_plain_form():
    from infernum_amd.kernels import api as K
    from infernum_amd.parts.softmax_attention import bias_by_distance
    T, H, G, d, dv, ps = 60, 6, 2, 20, 12, 4
    g = torch.Generator().manual_seed(1)
    q, k, v = torch.randn(T, H, d, generator=g), torch.randn(T, G, d, generator=g), torch.randn(T, G, dv, generator=g)
    rel, gate = torch.randn(10, H, generator=g), torch.randn(T, H * dv, generator=g)
    kp = k.view(T // ps, ps, G, d).permute(0, 2, 1, 3).contiguous().to(DEV)
    vp = v.view(T // ps, ps, G, dv).permute(0, 2, 3, 1).contiguous().to(DEV)
    out = torch.empty((T, H * dv), device=DEV)
    ar = torch.arange(T, dtype=torch.int32, device=DEV)
    K.attention_generic(q.reshape(T, -1).to(DEV), kp, vp, out, torch.zeros_like(ar), ar, ar[None, :T // ps].contiguous(), H, G, d, 0.4,
                        bias=K.distance_table(bias_by_distance(rel, 25.0)).to(DEV), gate=gate.to(DEV))
    want = MP.biased_attention(q.double(), k.double(), v.double(), 0.4, MP.distance_bias(T, rel.double(), 25.0)) * MP.sigmoid(gate.double())
    assert rel_err(out, want) <= 1e-5


# ------------------------------------------------------------------------------------ the recurrences' kernels
@BOTH
@pytest.mark.parametrize("dim,vdim,heads,rot", [(16, 16, 2, 16), (32, 64, 3, 8), (10, 6, 2, 0), (64, 128, 2, 64), (14, 9, 1, 6), (128, 128, 2, 128),
                                               (48, 80, 2, 20), (16, 256, 1, 0), (256, 32, 1, 24), (96, 192, 1, 96), (1, 1, 2, 0), (300, 520, 1, 100)])
def test_retention_at_many_head_sizes(dtype, dim, vdim, heads, rot):
    """Rows of unequal requests in one launch, from states that are not zero; then the same rows token by token (the same
    bits) and in tiles."""
    from infernum_amd.kernels import api as K
    rt = runtime(dtype)
    nq, nv = heads * dim, heads * vdim
    g = torch.Generator().manual_seed(dim)
    lens = [1, 40, 8, 2, 150, 64]
    N = sum(lens)
    row = -(-(2 * nq + 2 * nv) // 8) * 8
    proj = (torch.randn(N, row, generator=g)).to(rt.dtype)
    cols = (0, nq, 2 * nq, 2 * nq + nv)
    decay = [0.97, 0.0, 0.9990234375][:heads] if heads > 1 else [0.97]
    dec = torch.tensor([decay, [math.log2(x) if x else -math.inf for x in decay]], dtype=torch.float32).to(DEV)
    pos = torch.cat([torch.arange(n) + 5 * i for i, n in enumerate(lens)]).to(torch.int32)
    freq = (1000.0 ** (-2.0 * torch.arange(rot // 2, dtype=torch.float64) / rot)).to(DEV) if rot else None
    table = K.rotation_table(pos.to(DEV), freq) if rot else None
    slots = torch.tensor([3, 0, 2, 4, 6, 5], dtype=torch.int32)
    state = torch.randn(7, heads * dim * vdim, generator=g)
    starts = torch.tensor([0] + list(torch.tensor(lens).cumsum(0)), dtype=torch.int32)
    st, out = state.clone().to(DEV), torch.empty((N, nv), dtype=rt.dtype, device=DEV)
    args = (cols, table, rot, 0.3, dec, EPS, 1.5)
    sizes = (heads, dim, vdim)
    pd = proj.to(DEV)
    K.retention_step(pd, *args, st, out, starts.to(DEV), slots.to(DEV), *sizes)
    p64 = proj.double()
    q, k = p64[:, :nq].view(N, heads, dim), p64[:, nq:2 * nq].view(N, heads, dim)
    v, gt = p64[:, 2 * nq:2 * nq + nv].view(N, heads, vdim), p64[:, 2 * nq + nv:2 * nq + 2 * nv]
    if rot:
        q, k = MP.rotate_half(q, pos, rot, 1000.0), MP.rotate_half(k, pos, rot, 1000.0)
    want, want_state = torch.empty(N, heads, vdim, dtype=torch.float64), state.double().clone()
    for i, s in enumerate(slots.tolist()):
        lo, hi = int(starts[i]), int(starts[i + 1])
        for h in range(heads):
            o, S = MP.retention(q[lo:hi, h], 0.3 * k[lo:hi, h], v[lo:hi, h], decay[h], state.view(7, heads, dim, vdim)[s, h].double())
            want[lo:hi, h] = MP.unit_rms(o, EPS)
            want_state.view(7, heads, dim, vdim)[s, h] = S
    want = want.reshape(N, nv) * MP.silu(gt) * 1.5
    # a head that forgets at once is divided by a root mean square that can be small: the largest difference is allowed more
    tol = 5e-4 if dtype == "float32" else 1e-2
    assert rel_err(out, want) <= tol
    if dtype == "float32":
        assert (out.double().cpu() - want).pow(2).mean().sqrt() <= 1e-5 * want.pow(2).mean().sqrt()
    assert rel_err(st, want_state) <= 2e-5
    assert torch.equal(st[1].cpu(), state[1])                    # a slot that no request holds
    st2, out2 = state.clone().to(DEV), torch.empty_like(out)
    done = [0] * len(lens)
    while any(d < L for d, L in zip(done, lens)):
        live = [i for i in range(len(lens)) if done[i] < lens[i]]
        rows = torch.tensor([int(starts[i]) + done[i] for i in live])
        y = torch.empty((len(live), nv), dtype=rt.dtype, device=DEV)
        t = table[rows.to(DEV)].contiguous() if rot else None
        K.retention_step(pd[rows.to(DEV)].contiguous(), cols, t, *args[2:], st2, y,
                         torch.arange(len(live) + 1, dtype=torch.int32, device=DEV), slots[live].to(DEV), *sizes)
        out2[rows.to(DEV)] = y
        for i in live:
            done[i] += 1
    assert torch.equal(out, out2) and torch.equal(st, st2)
    if not K.retention_chunked_takes(rt.dtype, heads, dim, vdim, row, cols):
        return
    # in tiles, but for the first request's token, which a step brings alone; tiles in any order
    st3, out3 = state.clone().to(DEV), torch.full_like(out, 7.0)
    tiles = torch.tensor([(i, r) for i, L in list(enumerate(lens))[1:] for r in range(0, L, K.PREFILL_TILE_ROWS)][::-1], dtype=torch.int32)
    K.retention_chunked(pd, *args, st3, out3, starts.to(DEV), slots.to(DEV), tiles.to(DEV), tiles.shape[0], 1, *sizes)
    lo = lens[0]
    assert (out3[:lo] == 7).all()
    assert rel_err(out3[lo:], want[lo:]) <= 1e-2
    assert rel_err(st3, torch.where(torch.arange(7)[:, None] == slots[0], state.double(), want_state)) <= 2e-5


@BOTH
@pytest.mark.parametrize("C,Ns", [(64, 16), (96, 5), (50, 1), (130, 40), (200, 100), (256, 8), (33, 128), (512, 20)])
def test_selective_scan_at_many_sizes(dtype, C, Ns):
    """Rows of unequal requests in one launch, from states that are not zero; the same rows token by token (the same bits),
    and in segments of several lengths side by side."""
    from infernum_amd.kernels import api as K
    rt = runtime(dtype)
    g = torch.Generator().manual_seed(C)
    lens = [1, 1, 40, 8, 2, 150, 64]
    N, kn = sum(lens), K.selective_columns(Ns)
    x, z = _x(N, C, dtype, 1).to(rt.dtype), _x(N, C + 4, dtype, 2).to(rt.dtype)[:, :C]
    bc = torch.zeros(N, 8 + 2 * kn)
    bc[:, 8:8 + Ns], bc[:, 8 + kn:8 + kn + Ns] = torch.randn(N, Ns, generator=g), torch.randn(N, Ns, generator=g)
    bc = bc.to(rt.dtype)
    dt, bias = torch.randn(N, C, generator=g), torch.randn(C, generator=g) - 2.0
    A, D = -torch.exp(torch.randn(C, Ns, generator=g)), torch.randn(C, generator=g)
    a2 = (A * math.log2(math.e)).t().contiguous()
    slots = torch.tensor([3, 7, 0, 2, 4, 6, 5], dtype=torch.int32)
    state = torch.randn(8, Ns * C, generator=g)
    starts = torch.tensor([0] + list(torch.tensor(lens).cumsum(0)), dtype=torch.int32)
    want = torch.empty(N, C, dtype=torch.float64)
    want_state = state.double().clone()
    for i, s in enumerate(slots.tolist()):
        lo, hi = int(starts[i]), int(starts[i + 1])
        y, S = MP.selective_scan(x[lo:hi].double(), MP.softplus(dt[lo:hi].double() + bias.double()), A.double(), bc[lo:hi, 8:8 + Ns].double(),
                                 bc[lo:hi, 8 + kn:8 + kn + Ns].double(), D.double(), state[s].double().view(Ns, C).T)
        want[lo:hi], want_state[s] = y, S.T.reshape(-1)
    want = want * MP.silu(z.double())
    dev = [t.to(DEV) for t in (x, z, bc)]
    small = [t.to(DEV) for t in (dt, bias, a2, D)]
    tol = 3e-5 if dtype == "float32" else 1e-2

    def run(first, count, segment, st):
        out = torch.full((N, C), 7.0, dtype=rt.dtype, device=DEV)
        K.selective_scan(dev[0], dev[1], dev[2], 8, 8 + kn, *small, st, out, starts.to(DEV), slots.to(DEV), first, count, max(lens), segment)
        return out

    whole_state = state.clone().to(DEV)
    whole = run(0, 7, None, whole_state)
    assert rel_err(whole, want) <= tol and rel_err(whole_state, want_state) <= 2e-5
    assert torch.equal(whole_state[1].cpu(), state[1])
    for segment in (32, 64, 100):
        st = state.clone().to(DEV)
        out = run(2, 5, segment, st)
        assert (out[:2] == 7).all()
        assert rel_err(out[2:], want[2:]) <= tol and rel_err(st[[0, 2, 4, 5, 6]], want_state[[0, 2, 4, 5, 6]]) <= 2e-5, segment
        assert torch.equal(st[[1, 3, 7]].cpu(), state[[1, 3, 7]])
    st, out = state.clone().to(DEV), torch.empty((N, C), dtype=rt.dtype, device=DEV)
    done = [0] * len(lens)
    while any(d < L for d, L in zip(done, lens)):
        live = [i for i in range(len(lens)) if done[i] < lens[i]]
        rows = torch.tensor([int(starts[i]) + done[i] for i in live], device=DEV)
        y = torch.empty((len(live), C), dtype=rt.dtype, device=DEV)
        K.selective_scan(*[t[rows].contiguous() for t in dev], 8, 8 + kn, small[0][rows].contiguous(), *small[1:], st, y,
                         torch.arange(len(live) + 1, dtype=torch.int32, device=DEV), slots[live].to(DEV), 0, len(live), 1)
        out[rows] = y
        for i in live:
            done[i] += 1
    assert torch.equal(out, whole) and torch.equal(st, whole_state)


def test_where_rows_are_cut_into_segments():
    from infernum_amd.kernels import api as K
    assert K.selective_segment([40], 4096) == 40                               # short: in one piece
    assert K.selective_segment([256] * 64, 4096) == 256                        # many requests fill the GPU by themselves
    assert K.selective_segment([128] * 64, 4096) == 128
    assert K.selective_segment([8192], 4096) == 64                             # one long one is cut
    assert K.selective_segment([8000] + [3] * 60, 4096) == 64                  # also among many short ones
    assert K.selective_segment([300], 4096) == 32 and K.selective_segment([5000], 64) == 32
    assert K.selective_segment([], 64) == 1


# ------------------------------------------------------------------------------------ the mixers alone
SIDE_CASES = [(MM.V1["layers"][1]["mixer"], 64, 70), (MM.V1["layers"][3]["mixer"], 64, 45), (MM.V2["layers"][0]["mixer"], 100, 45),
              (MM.V2["layers"][2]["mixer"], 100, 33), (MM.V3["layers"][0]["mixer"], 128, 90), (MM.V5["layers"][0]["mixer"], 48, 60),
              (MM.V5["layers"][1]["mixer"], 48, 70)]
MAMBA_CASES = [(MM.V1["layers"][0]["mixer"], 64, 70), (MM.V2["layers"][1]["mixer"], 100, 45), (MM.V2["layers"][3]["mixer"], 100, 33),
               (MM.V3["layers"][1]["mixer"], 128, 90), (MM.V4["layers"][0]["mixer"], 80, 60), (MM.V4["layers"][1]["mixer"], 80, 40)]


@BOTH
@pytest.mark.parametrize("m,W,T", SIDE_CASES)
def test_both_mixers_side_by_side_and_each_alone(dtype, m, W, T):
    rt = runtime(dtype)
    tensors = _mixer_weights("parallel", m, W, 3)
    x = _x(T, W, dtype, 7)
    left = {k[5:]: v for k, v in tensors.items() if k.startswith("left.")}
    right = {k[6:]: v for k, v in tensors.items() if k.startswith("right.")}
    cases = [("softmax_attention", _left_params(m["left"], W), left, lambda w, r: MP.attention_mixer(x.double(), w, "", m["left"], EPS, r)),
             ("retention", _right_params(m["right"], W), right, lambda w, r: MP.retention_mixer(x.double(), w, "", m["right"], EPS, r)),
             ("side_by_side", _side_params(m, W), tensors, lambda w, r: MP.parallel_mixer(x.double(), w, "", m, EPS, r))]
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
                steps.cache.release(f"r{i}")
                steps.cache.check()
                assert rel_err(got.to(rt.dtype), want) <= tol, (kind, ps, cuts[:3])


@BOTH
@pytest.mark.parametrize("m,W,T", MAMBA_CASES)
def test_selective_scan_mixer_alone(dtype, m, W, T):
    rt = runtime(dtype)
    mixer, w = _build("mamba1", _mamba_params(m, W), rt, _mixer_weights("mamba1", m, W, 3))
    x = _x(T, W, dtype, 7)
    want = MP.mamba_mixer(x.double(), w, "", m, EPS)
    tol = _tol(dtype, want, lambda: MP.mamba_mixer(x.double(), w, "", m, EPS, torch.bfloat16))
    steps = _steps_for(mixer, rt, 16, 12, slots=2)
    for i, cuts in enumerate(CUTS(T)):
        got = _run_mixer(mixer, steps, x, cuts, rt, request=f"r{i}")
        steps.cache.release(f"r{i}")
        assert rel_err(got.to(rt.dtype), want) <= tol, cuts[:3]


@BOTH
@pytest.mark.parametrize("rows,far", [(6, 9.5), (20, 40.0), (64, 300.0), (2, 3.0)])
def test_every_edge_of_the_bias_by_distance(dtype, rows, far):
    """Scores of nothing but the bias, whose rows take turns between +4 and -4, and values that tell a key's place: a key
    counted into the wrong row shows.  Whole, decoded, in portions that begin anywhere, pages of 4 and 16."""
    T, W = 150, 32
    rt = runtime(dtype)
    m = {"heads": 2, "kv_heads": 1, "dim": 16, "vdim": 16, "scale": 0.25, "bias_max": far, "buckets": rows}
    w = _mixer_weights("parallel", {"left": m, "right": MM._right(1, 16, 16, [0.5]), "left_scale": 1, "right_scale": 1}, W, 3)
    w = {k[5:]: v for k, v in w.items() if k.startswith("left.")}
    w["q"] = w["q"] * 0.0
    w["rel"] = (4.0 * (1.0 - 2.0 * (torch.arange(rows) % 2)))[:, None] * torch.tensor([[1.0, -1.0]])
    w["rel"] = w["rel"].double()
    mixer, w = _build("softmax_attention", _left_params(m, W), rt, w)
    x = _x(T, W, dtype, 9)
    want = MP.attention_mixer(x.double(), w, "", m, EPS)
    off = dict(w, rel=w["rel"].roll(1, 0))
    assert rel_err(MP.attention_mixer(x.double(), off, "", m, EPS), want) > 0.5
    tol = _tol(dtype, want, lambda: MP.attention_mixer(x.double(), w, "", m, EPS, torch.bfloat16))
    for ps in (4, 16):
        for cuts in CUTS(T):
            got = _run_mixer(mixer, _steps_for(mixer, rt, ps, T // ps + 2), x, cuts, rt)
            assert rel_err(got.to(rt.dtype), want) <= tol, (ps, cuts[:3])


@BOTH
@pytest.mark.parametrize("star", [0, 2, 15, 16, 63])
def test_a_key_far_back_among_hundreds(dtype, star):
    """One key alone points the queries' way and answers them 500 positions later, across the far end of the bias."""
    T, W, d = 540, 8, 16
    rt = runtime(dtype)
    m = {"heads": 1, "kv_heads": 1, "dim": d, "vdim": d, "scale": 1.0, "bias_max": 30.0, "buckets": 8}
    z = lambda *s: torch.zeros(s, dtype=torch.float64)          # noqa: E731
    w = {"q": z(d, W), "k": z(d, W), "v": z(d, W), "g": z(d, W), "o": z(W, d), "q.norm": torch.ones(d), "k.norm": torch.ones(d),
         "rel": torch.linspace(0.0, -2.0, 8)[:, None]}
    w["q"][0, 0] = 1.0
    w["k"][0, 1], w["k"][1, 2] = 1.0, 1.0
    w["v"][0, 1] = 10.0
    w["o"][0, 0] = 1.0
    x = torch.zeros(T, W)
    x[:, 0], x[:, 2] = 1.0, 1.0
    x[star, 1], x[star, 2] = 1.0, 0.0
    mixer, w = _build("softmax_attention", _left_params(m, W), rt, w)
    want = MP.attention_mixer(x.double(), w, "", m, EPS)
    assert (want[star:, 0] > 4.0).all() and (want[:star, 0].abs() < 0.1).all()
    tol = _tol(dtype, want, lambda: MP.attention_mixer(x.double(), w, "", m, EPS, torch.bfloat16))
    for cuts in ([T], [T - 20] + [1] * 20, [63, 2, 100, 64, 1, 2, T - 232]):
        got = _run_mixer(mixer, _steps_for(mixer, rt, 16, T // 16 + 2), x, cuts, rt)
        assert rel_err(got.to(rt.dtype), want) <= tol, cuts[:2]


@BOTH
def test_states_that_reach_hundreds_of_tokens_back(dtype):
    """What token 3 wrote is read 600 tokens later: by a retention head that never forgets (beside one that does), and by
    channels of the selective scan whose steps are small; whole and decoded."""
    T, W = 640, 32
    rt = runtime(dtype)
    x = _x(T, W, dtype, 11)
    x[:, 0], x[:, 1] = 0.0, 1.0
    x[3, 0] = 40.0
    other = x.clone()
    other[3, 0] = 0.0
    m = {"heads": 2, "dim": 16, "vdim": 16, "decay": [1.0, 0.5]}
    p = {"left": MM._left(1, 1, 16, 16, 1.0, 20.0, 8), "right": m, "left_scale": 1.0, "right_scale": 1.0}
    w = {k[6:]: v for k, v in _mixer_weights("parallel", p, W, 5).items() if k.startswith("right.")}
    w["k"][:, 1:] = 0.02 * w["k"][:, 1:]
    w["q"][:16] = 0.0
    w["q"][:16, 1] = w["k"][:16, 0]
    cases = [("retention", _right_params(m, W), w, lambda a, w, r=None: MP.retention_mixer(a, w, "", m, EPS, r))]
    mm = MM._mamba(48, 16, 4, 4)
    w = _mixer_weights("mamba1", mm, W, 5)
    w["dt.b"], w["A_log"] = w["dt.b"] * 0.0 - 1.0, w["A_log"] * 0.0 - 8.0
    w["dt"] = 0.1 * w["dt"]
    cases.append(("mamba1", _mamba_params(mm, W), w, lambda a, w, r=None: MP.mamba_mixer(a, w, "", mm, EPS, r)))
    for kind, params, ts, plain in cases:
        mixer, w = _build(kind, params, rt, ts)
        want = plain(x.double(), w)
        tol = _tol(dtype, want, lambda: plain(x.double(), w, torch.bfloat16))
        if dtype == "float32":
            tol = max(tol, 8.0 * rel_err(plain(x.double(), w, torch.float32), want))
        reach = (want[-1] - plain(other.double(), w)[-1]).abs().max() / want.pow(2).mean().sqrt()
        assert reach > 5e-2, (kind, float(reach))
        if dtype == "bfloat16":
            tol = min(tol, 0.5 * float(reach))
        for cuts in ([T], [300, 209, 1, 1, 1, 1, 1, T - 514], [3, 1, T - 10] + [1] * 6):
            got = _run_mixer(mixer, _steps_for(mixer, rt, 16, 4, slots=2),
                             x, cuts, rt)
            assert rel_err(got.to(rt.dtype), want) <= tol, (kind, cuts[:2])


@BOTH
@pytest.mark.parametrize("mlp,W,N", [(MM.V1["layers"][0]["mlp"], 64, 60), (MM.V2["layers"][0]["mlp"], 100, 9), (MM.V2["layers"][3]["mlp"], 100, 40),
                                     (MM.V3["layers"][1]["mlp"], 128, 1), (MM.V4["layers"][0]["mlp"], 80, 30), (MM.V5["layers"][1]["mlp"], 48, 70),
                                     (MM._moe(64, 4, 2, 64), 64, 300), (MM._moe(64, 6, 3), 128, 400)])
def test_routed_experts_with_weights_on_their_inputs(dtype, mlp, W, N):
    """Few tokens and so many that the grouped product takes them; places where the choice is no close call."""
    rt = runtime(dtype)
    layer = {"type": "mamba1", "mixer": MM._mamba(4, 1, 1, 1), "mlp": mlp}
    ts = {k[4:]: v for k, v in _layer_weights(layer, W, 8).items() if k.startswith("mlp.")}
    part, w = _build("routed_experts", {
        "hidden_size": W, "intermediate_size": mlp["expert"]["ff"], "num_experts": mlp["router"]["experts"], "top": mlp["router"]["top"],
        "gated": True, "limit": None, "alpha": 1.0, "up_shift": 0.0, "router": "softmax_top", "scores": "sigmoid", "renorm": False,
        "correction_name": None, "weights_on": "input", "shared_ff": (mlp.get("shared") or {}).get("ff")}, rt, ts, "feed_forward")
    x = _x(N, W, dtype, 9)
    margins = []
    want = MP.routed_experts(x.double(), w, "", mlp, margins=margins)
    sure = margins[0] > 3e-4
    assert sure.sum() >= 0.7 * N
    rounded = MP.routed_experts(x.double(), w, "", mlp, torch.bfloat16)
    got = dense(part.forward(x.to(DEV).to(rt.dtype)), rt).cpu()
    assert torch.isfinite(got.float()).all()
    assert rel_err(got[sure], want[sure]) <= _tol(dtype, want[sure], lambda: rounded[sure])


@BOTH
@pytest.mark.parametrize("kind", ["side_by_side", "mamba1"])
def test_requests_of_unequal_length_side_by_side_and_alone(dtype, kind):
    """A batch of unequal requests in steps of unequal portions: every row as if its request were alone."""
    W = 64
    m = MM.V1["layers"][1 if kind == "side_by_side" else 0]["mixer"]
    plain = (lambda a, w, r=None: MP.parallel_mixer(a, w, "", m, EPS, r)) if kind == "side_by_side" else \
        (lambda a, w, r=None: MP.mamba_mixer(a, w, "", m, EPS, r))
    rt = runtime(dtype)
    mixer, w = _build(kind, _side_params(m, W) if kind == "side_by_side" else _mamba_params(m, W), rt,
                      _mixer_weights("parallel" if kind == "side_by_side" else "mamba1", m, W, 4))
    lens = {"a": 1, "b": 130, "c": 64, "d": 65, "e": 1, "f": 7}
    xs = {r: _x(n + 3, W, dtype, 20 + i) for i, (r, n) in enumerate(lens.items())}
    want = {r: plain(x.double(), w) for r, x in xs.items()}
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
        tol = _tol(dtype, want[r], lambda: plain(xs[r].double(), w, torch.bfloat16))
        if dtype == "float32":
            tol = max(tol, 8.0 * rel_err(plain(xs[r].double(), w, torch.float32), want[r]))
        assert rel_err(torch.cat(got[r]).to(rt.dtype), want[r]) <= tol, r


# ------------------------------------------------------------------------------------ the engine
TOLERANCE = {}


def _requests(cfg, w, lengths, seed, margins=None):
    reqs = TT.make_requests(cfg["vocab"], lengths, seed=seed)
    return reqs, {r: MP.forward(cfg, w, t, margins=margins) for r, t in reqs.items()}


class _Model:
    """A model folder per compute type.  In 32-bit the routers are random (no choice of the requests is closer than rounding
    can turn); in bfloat16 they read levels far apart."""

    def __init__(self, name, root):
        self.name, self.cfg = name, MM.RAW[name]
        natural = MP.random_weights(self.cfg, MM.SEED[name])
        self.w = {"float32": natural, "bfloat16": MM.decided(self.cfg, natural)}
        self.dir, self.reqs, self.ref, self.mreqs, self.mref = {}, None, {}, None, {}
        for dtype, w in self.w.items():
            self.dir[dtype] = str(root / dtype)
            MM.write_model(self.cfg, self.dir[dtype], weights=w)
            margins = [torch.ones(1)]
            self.reqs, self.ref[dtype] = _requests(self.cfg, w, LENGTHS[name], 11, margins)
            self.mreqs, self.mref[dtype] = _requests(self.cfg, w, MIXED[name], 23, margins)
            assert min(float(m.min()) for m in margins) > (1e-5 if dtype == "float32" else 1e-2)
            to = torch.bfloat16 if dtype == "bfloat16" else torch.float32
            cost = 0.0
            for group, refs in ((self.reqs, self.ref[dtype]), (self.mreqs, self.mref[dtype])):
                for r, t in group.items():
                    cost = max(cost, (MP.forward(self.cfg, w, t, round_to=to) - refs[r]).abs().max().item() / refs[r].pow(2).mean().sqrt().item())
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
    """The logits of the models made of the first k layers, one pass each (the same tensors), k = 1, 2, ...: a layer that
    differs shows at its own k.  The parts' own way gives what the step's program gives."""
    import copy
    from infernum_amd.engine import StepEntry
    m = models[name]
    toks = m.reqs["r2"]
    for k in range(1, len(m.cfg["layers"]) + 1):
        sub = copy.deepcopy(m.cfg)
        sub["layers"] = sub["layers"][:k]
        sub.pop("loop", None)
        keep = {n: t for n, t in m.w[dtype].items()
                if n != "loop.step" and (not (n[0] == "l" and n[1].isdigit()) or int(n[1:n.index(".")]) < k)}
        sd = str(tmp_path / f"first{k}")
        MM.write_model(sub, sd, weights=keep)
        logits = _engine(sd, dtype, PAGE[name], 64).step([StepEntry("a", toks, list(range(len(toks))))]).cpu()
        _check({("a", p): logits[p] for p in range(len(toks))}, {"a": MP.forward(sub, keep, toks)}, dtype,
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
        assert all(rel_err(got[k], alone[k].cpu()) <= 2e-5 for k in got)


@BOTH
@pytest.mark.parametrize("name", ["V1", "V3", "V4"])
def test_long_decoding(models, name, dtype):
    """A short prompt, then 150 tokens one by one: the states move on 150 times, the bias passes over decoded tokens, pages
    fill and begin; decode steps are replayed from graphs after the first two."""
    m = models[name]
    w = m.w[dtype]
    reqs, ref = _requests(m.cfg, w, (160,), 3)
    cost = max((MP.forward(m.cfg, w, t, round_to=torch.float32 if dtype == "float32" else torch.bfloat16) - ref[r]).abs().max().item()
               / ref[r].pow(2).mean().sqrt().item() for r, t in reqs.items())
    TOLERANCE[name, dtype] = max(TOLERANCE[name, dtype], (8.0 if dtype == "float32" else 3.0) * cost)
    eng = _engine(m.dir[dtype], dtype, 16, 12)
    _check(TT.run_steps(eng, TT.trace_tail_one_by_one(reqs, 150)), ref, dtype, f"{name} {dtype} long decoding", name)
    assert eng.graph_replays > 100


def test_greedy_generation_through_the_scheduler(models):
    """Runtime.generate_batch (scheduler, portions, the sampler's argmax) against the plain model's greedy tokens,
    in 32-bit; prompts of unequal length, more requests than run at once."""
    from infernum_amd import BatchConfig, GenerateOptions, Runtime
    m = models["V1"]
    prompts = list(TT.make_requests(m.cfg["vocab"], (5, 31, 2, 18, 9), seed=9).values())
    rt = Runtime.from_pretrained(m.dir["float32"], dtype="float32",
                                 batch_config=BatchConfig(block_size=16, num_blocks=24, max_batch_size=3, max_prefill_tokens=8,
                                                          max_tokens_per_step=16, step_token_multiple=1))
    outs = rt.generate_batch(prompts, GenerateOptions(max_new_tokens=12))
    for p, got in zip(prompts, outs):
        toks = list(p)
        for _ in range(12):
            toks.append(int(MP.forward(m.cfg, m.w["float32"], toks)[-1].argmax()))
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
    m = models["V3"]
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
    _check(got, m.mref[dtype], dtype, f"trace_run V3 {dtype} mixed", "V3")
    if dtype == "float32":
        prompt = reqs["r4"][:9]
        gen = subprocess.run([sys.executable, os.path.join(root, "bin", "generate"), "-m", m.dir[dtype], "--prompt-ids",
                              ",".join(map(str, prompt)), "-n", "6", "--greedy", "--dtype", "float32"],
                             text=True, capture_output=True, timeout=100)
        assert gen.returncode == 0, gen.stderr[-3000:]
        toks = list(prompt)
        for _ in range(6):
            toks.append(int(MP.forward(m.cfg, m.w[dtype], toks)[-1].argmax()))
        assert " " + " ".join(map(str, toks[9:])) + "\n" in gen.stdout, gen.stdout[-2000:]
