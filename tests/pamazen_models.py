"""Small Pamazen configurations for the tests, and a helper that writes their model folders from the plain
implementation's random weights.

P1: both mixers, three streams; the side-by-side layer with six query heads over two, a window of 20 with 3 kept
    positions and a softcap; half-rotated heads whose values are smaller than their keys; three layers that mix values;
    eight experts of which two are identities, in four groups of which two are kept.
P2: sizes that no fast kernel takes (width 100, odd vocabulary, heads of 20 and of 12 with values of 10, a recurrence
    of heads of 10, a middle of 7); a window of 7 that keeps 5; as many key/value heads as heads; a layer without
    experts; no groups, no identity experts, no shared expert, one expert a token; no rotation in one layer; no caps;
    two streams.
P3: five streams; twenty heads over one key/value head; a window of 1 that keeps 17 positions (more than a page); a
    window of 48 that keeps one; values larger than their keys; a value-mixing layer before and after one that does not
    mix; every group kept; wide correction.
P4: side-by-side layers only; one stream; a window that keeps nothing; no window at all; heads of 40 in the recurrence.
P5: attention layers only (no state slot at all); nine streams; a whole head rotated with the plain frequencies; the last
    layer has no experts; the residual multiplier is 1.
"""
import json
import os

import plain_pamazen as PP


def _rot(base, dims, factor=None):
    r = {"base": base, "dims": dims}
    if factor is not None:
        r["scaling"] = {"factor": factor}
    return r


def _attn(heads, kv_heads, dim, vdim, scale, rot=None, v_mix=False):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "v_mix": v_mix}
    if rot is not None:
        m["rot"] = rot
    return m


def _left(heads, kv_heads, dim, scale, size=None, keep=0, cap=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if cap is not None:
        m["softcap"] = cap
    if size is not None:
        m["mask"] = {"size": size, "keep_first": keep}
    return m


def _par(left, heads, dim, ls, rs):
    return {"left": left, "right": {"heads": heads, "dim": dim}, "left_scale": ls, "right_scale": rs}


def _moe(ff, experts, top, identity=0, groups=None, shared=None):
    r = {"experts": experts, "identity": identity, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    out = {"kind": "moe", "expert": {"ff": ff}, "router": r}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def _layer(kind, mixer, mlp=None):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


_m1 = _moe(32, 6, 3, 2, (4, 2), 48)
P1 = {"architecture": "Pamazen", "vocab": 200, "width": 64, "norm": {"eps": 1e-5}, "streams": 3, "residual_mult": 0.4,
      "logit_softcap": 9.0,
      "layers": [_layer("parallel", _par(_left(6, 2, 32, 0.2, 20, 3, 7.0), 3, 16, 0.9, 0.6), _m1),
                 _layer("attention", _attn(4, 2, 32, 16, 0.2, _rot(10000.0, 16, 2.0), True), _m1),
                 _layer("attention", _attn(4, 2, 32, 16, 0.25, _rot(500.0, 32, 3.0), True), _m1),
                 _layer("parallel", _par(_left(4, 4, 16, 0.3, 33, 2, 20.0), 2, 32, 1.3, 0.7), _m1),
                 _layer("attention", _attn(6, 1, 16, 32, 0.25, _rot(10000.0, 8, 4.0), True), _moe(64, 6, 2, 2, (2, 1), 64))]}
P2 = {"architecture": "Pamazen", "vocab": 333, "width": 100, "norm": {"eps": 1e-6}, "streams": 2, "residual_mult": 0.7,
      "layers": [_layer("parallel", _par(_left(5, 5, 20, 0.25, 7, 5), 2, 10, 1.1, -0.5), _moe(20, 5, 1)),
                 _layer("attention", _attn(3, 3, 12, 10, 0.35, _rot(1000.0, 6)), None),
                 _layer("attention", _attn(4, 2, 20, 15, 0.25, None, True), _moe(30, 4, 2, 3, None, 12))]}
P3 = {"architecture": "Pamazen", "vocab": 256, "width": 128, "norm": {"eps": 3e-6}, "streams": 5, "residual_mult": 0.3,
      "logit_softcap": 30.0,
      "layers": [_layer("attention", _attn(4, 2, 16, 48, 0.3, _rot(10000.0, 16, 8.0), True), _moe(64, 10, 4, 2, (3, 3), 32)),
                 _layer("parallel", _par(_left(20, 1, 32, 0.2, 1, 17, 15.0), 4, 64, 0.7, 1.2), _moe(64, 12, 2, 4, (8, 3), 64)),
                 _layer("attention", _attn(8, 2, 64, 64, 0.125, _rot(20000.0, 24, 1.5)), _moe(64, 10, 4, 2, (3, 1))),
                 _layer("attention", _attn(3, 3, 48, 32, 0.15, _rot(10000.0, 48, 2.0), True), None),
                 _layer("parallel", _par(_left(4, 2, 48, 0.15, 48, 1, 5.0), 1, 96, 1.0, 0.4), _moe(32, 2, 1, 1, None, 32))]}
P4 = {"architecture": "Pamazen", "vocab": 150, "width": 80, "norm": {"eps": 1e-5}, "streams": 1, "residual_mult": 0.5,
      "logit_softcap": 15.0,
      "layers": [_layer("parallel", _par(_left(2, 1, 16, 0.3, 25, 0, 6.0), 5, 16, 0.5, 1.5), _moe(32, 3, 2, 1, (2, 1), 16)),
                 _layer("parallel", _par(_left(4, 2, 32, 0.2), 2, 40, 1.0, 1.0), _moe(48, 4, 2))]}
P5 = {"architecture": "Pamazen", "vocab": 1100, "width": 48, "norm": {"eps": 1e-5}, "streams": 9, "residual_mult": 1.0,
      "layers": [_layer("attention", _attn(3, 3, 48, 16, 0.15, _rot(10000.0, 48)), _moe(16, 7, 3, 1, (4, 3), 24)),
                 _layer("attention", _attn(4, 2, 16, 16, 0.25, _rot(300000.0, 8, 3.0), True), _moe(32, 3, 3)),
                 _layer("attention", _attn(2, 1, 64, 32, 0.1, None, True), None)]}
RAW = {"P1": P1, "P2": P2, "P3": P3, "P4": P4, "P5": P5}
SEED = {"P1": 5, "P2": 6, "P3": 7, "P4": 15, "P5": 9}


def decided(cfg, w, seed=0):
    """The same weights with corrections so far apart that they alone decide which experts (and groups) a layer's tokens
    take: no rounding can turn a choice.  The weights of the chosen still come from the router."""
    import torch
    g = torch.Generator().manual_seed(seed)
    out = dict(w)
    for n, t in w.items():
        if n.endswith("mlp.correction"):
            out[n] = (2.0 * torch.randperm(t.numel(), generator=g).to(torch.float32) - 4.0).to(t.dtype)
    return out


def write_model(name_or_cfg, out_dir: str, seed=None, weights=None):
    """Writes config.json and model.safetensors (bfloat16 values); returns (configuration dict, weights dict) as
    the plain implementation reads them."""
    import torch
    from infernum_amd.weights.safetensors_io import write_safetensors
    cfg = RAW[name_or_cfg] if isinstance(name_or_cfg, str) else name_or_cfg
    seed = (SEED[name_or_cfg] if isinstance(name_or_cfg, str) else 0) if seed is None else seed
    w = weights if weights is not None else PP.random_weights(cfg, seed)
    os.makedirs(out_dir, exist_ok=True)
    with open(os.path.join(out_dir, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(out_dir, "model.safetensors"),
                      ((n, t.to(torch.bfloat16).contiguous()) for n, t in sorted(w.items())))
    return cfg, w
