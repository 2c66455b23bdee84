"""Small Mirovik configurations for the tests, and a helper that writes their model folders from the plain
implementation's random weights.

V1: both mixers; four query heads over two with values smaller than keys, a bias table of 20 rows up to 40 places back, three
    retention heads whose values are larger than their keys, half of a head rotated; two of six experts and a shared one;
    a dense middle; the two middle layers run twice.
V2: sizes that no fast kernel takes (width 100, odd vocabulary, heads of 20 and 12, retention heads of 10 and 6, a state of
    5); as many key/value heads as heads; a bias table of 6 rows up to 9.5 places; no rotation; a convolution of one tap; a
    layer without a feed-forward; no repetition, the table's rows as they are.
V3: twenty heads over one key/value head; a bias that grows up to 300 places, further than any request is long; one retention
    head of 64 and 128 that never forgets, all of it rotated; a state of 40, a convolution of two taps; three of five experts
    without a shared one; the whole model runs three times.
V4: the selective scan only (no pages at all); a state of one value; a single expert; the last layer runs four times.
V5: side-by-side layers only; values larger than keys; a bias table of two rows; retention heads that forget at once (decay
    0), fast and slowly; the repeated stretch is one pass.
"""
import json
import os

import plain_mirovik as MP


def _left(heads, kv_heads, dim, vdim, scale, bias_max, buckets):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "bias_max": bias_max, "buckets": buckets}


def _right(heads, dim, vdim, decay, rot=None):
    r = {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}
    if rot:
        r["rot"] = {"base": rot[0], "dims": rot[1]}
    return r


def _par(left, right, ls, rs):
    return {"left": left, "right": right, "left_scale": ls, "right_scale": rs}


def _mamba(inner, state, dt_rank, conv):
    return {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(ff, experts, top, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def _layer(kind, mixer, mlp=None):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


_P, _M = "parallel", "mamba1"
V1 = {"architecture": "Mirovik", "vocab": 200, "width": 64, "norm": {"eps": 1e-5}, "embedding": {"scale": 8.0},
      "loop": {"start": 1, "stop": 3, "times": 2},
      "layers": [_layer(_M, _mamba(96, 16, 5, 4), _moe(32, 6, 2, 48)),
                 _layer(_P, _par(_left(4, 2, 32, 16, 0.25, 40.0, 20), _right(3, 16, 32, [0.9, 0.96875, 0.998], (10000.0, 8)), 0.8, 1.3), _dense(96)),
                 _layer(_M, _mamba(128, 8, 12, 3), _moe(64, 6, 2, 64)),
                 _layer(_P, _par(_left(6, 3, 16, 16, 0.4, 30.0, 14), _right(2, 32, 16, [0.5, 0.99], (500.0, 32)), 1.1, 0.6), _moe(32, 4, 1))]}
V2 = {"architecture": "Mirovik", "vocab": 333, "width": 100, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
      "layers": [_layer(_P, _par(_left(3, 3, 20, 12, 0.3, 9.5, 6), _right(2, 10, 6, [0.75, 0.99609375]), 1.1, -0.5), _moe(20, 5, 3)),
                 _layer(_M, _mamba(50, 5, 3, 1), None),
                 _layer(_P, _par(_left(4, 2, 12, 20, 0.35, 50.0, 10), _right(3, 14, 9, [0.2, 1.0, 0.97], (1000.0, 6)), 0.7, 0.9), _dense(60)),
                 _layer(_M, _mamba(66, 20, 7, 5), _moe(30, 3, 1, 12))]}
V3 = {"architecture": "Mirovik", "vocab": 256, "width": 128, "norm": {"eps": 3e-6}, "embedding": {"scale": 11.0},
      "loop": {"start": 0, "stop": 2, "times": 3},
      "layers": [_layer(_P, _par(_left(20, 1, 16, 16, 0.3, 300.0, 64), _right(1, 64, 128, [1.0], (20000.0, 64)), 1.0, 0.7), _dense(64)),
                 _layer(_M, _mamba(72, 40, 9, 2), _moe(64, 5, 3))]}
V4 = {"architecture": "Mirovik", "vocab": 150, "width": 80, "norm": {"eps": 1e-5}, "embedding": {"scale": 9.0},
      "loop": {"start": 2, "stop": 3, "times": 4},
      "layers": [_layer(_M, _mamba(32, 1, 1, 4), _moe(32, 1, 1, 16)), _layer(_M, _mamba(200, 100, 16, 3), None),
                 _layer(_M, _mamba(160, 12, 6, 4), _dense(112))]}
V5 = {"architecture": "Mirovik", "vocab": 1100, "width": 48, "norm": {"eps": 1e-5}, "embedding": {"scale": 7.0},
      "loop": {"start": 1, "stop": 2, "times": 1},
      "layers": [_layer(_P, _par(_left(3, 3, 48, 80, 0.15, 3.0, 2), _right(3, 32, 16, [0.0, 0.1, 0.9990234375], (3000.0, 16)), 1.5, 0.0625), _dense(64)),
                 _layer(_P, _par(_left(2, 1, 64, 64, 0.2, 33.0, 16), _right(2, 16, 48, [0.8, 0.95], (10000.0, 16)), 0.6, 1.0), _moe(16, 7, 3, 24)),
                 _layer(_P, _par(_left(4, 2, 16, 16, 0.5, 64.0, 32), _right(1, 48, 64, [0.99]), 1.0, 1.0), None)]}
RAW = {"V1": V1, "V2": V2, "V3": V3, "V4": V4, "V5": V5}
SEED = {"V1": 12, "V2": 10, "V3": 7, "V4": 8, "V5": 9}


def decided(cfg, w, seed=0):
    """The same weights with routers that no rounding can turn: the first places of a token's embedding hold levels far
    apart in an order of the token's own, no sublayer writes to those places (the norm behind it is zero there), and the
    routers read them alone.  Which experts a token takes still varies, and so do the scores."""
    import torch
    experts = [l["mlp"]["router"]["experts"] for l in cfg["layers"] if l.get("mlp") and l["mlp"]["kind"] == "moe"]
    if not experts:
        return dict(w)
    D, g = max(experts), torch.Generator().manual_seed(seed)
    out = {n: t.clone() for n, t in w.items()}
    order = torch.stack([torch.randperm(D, generator=g) for _ in range(cfg["vocab"])]).float()
    out["embed"][:, :D] = ((2.0 * (order + 0.5) / D - 1.0) * 4.0 / float((cfg.get("embedding") or {}).get("scale", 1.0))).to(out["embed"].dtype)
    for n, t in out.items():
        if n.endswith((".norm1b", ".norm2b")):
            t[:D] = -1.0
        elif n.endswith(".norm2"):
            t[:D] = 0.0
        elif n == "loop.step":
            t[:, :D] = 0.0
        elif n.endswith(".router"):
            t.zero_()
            t[:, :t.shape[0]] = 3.0 * torch.eye(t.shape[0]).to(t.dtype)
    return out


def write_model(name_or_cfg, out_dir: str, seed=None, weights=None):
    """Writes config.json and model.safetensors (bfloat16 values); returns (configuration dict, weights dict) as
    the plain implementation reads them."""
    import torch
    from infernum_amd.weights.safetensors_io import write_safetensors
    cfg = RAW[name_or_cfg] if isinstance(name_or_cfg, str) else name_or_cfg
    seed = (SEED[name_or_cfg] if isinstance(name_or_cfg, str) else 0) if seed is None else seed
    w = weights if weights is not None else MP.random_weights(cfg, seed)
    os.makedirs(out_dir, exist_ok=True)
    with open(os.path.join(out_dir, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(out_dir, "model.safetensors"),
                      ((n, t.to(torch.bfloat16).contiguous()) for n, t in sorted(w.items())))
    return cfg, w
