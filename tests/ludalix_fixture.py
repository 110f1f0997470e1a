"""Small random Ludalix models for the tests: layer descriptions, tensor shapes, weights that are exact in bf16."""
from __future__ import annotations

import numpy as np

import ludalix_oracle as lo
from block_fixture import bf16, build, error  # noqa: F401


def dense(ff=50, limit=1.2):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts=5, top=2, ff=23):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def attn(heads=6, kv_heads=2, dim=20, vdim=14, window=25, keep=3, scale=0.21, kv_from=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if window:
        m["mask"] = {"size": window, "keep_first": keep}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": mlp}


def memory(heads=3, dim=20, vdim=26, cap=7.0, mlp=None):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": mlp}


def config(layers, width=72, vocab=101, scale=5.5, eps=3e-5, mult=0.4):
    return {"architecture": "Ludalix", "embedding": {"scale": scale}, "layers": list(layers), "norm": {"eps": eps}, "residual_mult": mult,
            "vocab": vocab, "width": width}


def shapes(cfg):
    """name -> shape of every tensor the configuration calls for."""
    W, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}
    for i, l in enumerate(cfg["layers"]):
        m, p, x, H = l["mixer"], f"l{i}.", f"l{i}.mix.", l["mixer"]["heads"]
        out[p + "norm1"] = (W,)
        if l["type"] == "attention":
            out |= {x + "q": (H * m["dim"], W), x + "q.norm": (m["dim"],), x + "o": (W, H * m["vdim"])}
            if "kv_from" not in m:
                out |= {x + "k": (m["kv_heads"] * m["dim"], W), x + "k.norm": (m["dim"],), x + "v": (m["kv_heads"] * m["vdim"], W)}
        else:
            hv = H * m["vdim"]
            out |= {x + "q": (H * m["dim"], W), x + "k": (H * m["dim"], W), x + "v": (hv, W), x + "g": (hv, W), x + "o": (W, hv), x + "norm": (hv,)}
            out |= {x + "i": (H, W), x + "i.b": (H,), x + "f": (H, W), x + "f.b": (H,)}
        mlp = l["mlp"]
        if not mlp:
            continue
        out[p + "norm2"] = (W,)
        many = mlp["kind"] == "moe"
        ff = mlp["expert"]["ff"] if many else mlp["ff"]
        for e in range(mlp["router"]["experts"]) if many else [None]:
            y = p + "mlp." + (f"e{e}." if many else "")
            out |= {y + "gate": (ff, W), y + "up": (ff, W), y + "down": (W, ff)}
        if many:
            out[p + "mlp.router"] = (mlp["router"]["experts"], W)
    return out | {"final.norm": (W,), "head": (cfg["vocab"], W)}


def weights(cfg, seed=0, gates=(0.0, 2.0)):
    """gates: means of the input and the forget gates' biases."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in shapes(cfg).items():
        z = rng.standard_normal(shape)
        if "norm" in name.split(".")[-1]:
            w = 1.0 + 0.25 * z
        elif name.endswith(".b"):
            w = gates[name.endswith("f.b")] + z
        elif name == "embed":
            w = z
        elif name.split(".")[-1] in ("q", "k", "v", "g", "i", "f", "gate", "up", "router"):
            w = z / np.sqrt(shape[-1]) / (0.5 * cfg["embedding"]["scale"])  # these read the residual itself
        else:
            w = z / np.sqrt(shape[-1])
        out[name] = bf16(w)
    return out


def clearest(cfg, n, seeds, gates=(0.0, 2.0)):
    """(weights, tokens) among a few seeds whose experts' choices are least close: at reduced precision a close call may
    fall the other way, which says nothing about the computation."""
    best = None
    for seed in seeds:
        w, toks = weights(cfg, seed, gates), np.random.default_rng(seed + 1).integers(0, cfg["vocab"], n)
        margins, route = [1.0], lo.route

        def watched(h, router, top):
            z = h @ router.T
            if top < z.shape[1]:
                s = -np.sort(-z, axis=1)
                margins.append(float(((s[:, top - 1] - s[:, top]) / z.std()).min()))
            return route(h, router, top)

        lo.route = watched
        try:
            want, trail = lo.forward(cfg, w, toks)
        finally:
            lo.route = route
        if best is None or min(margins) > best[0]:
            best = (min(margins), w, toks, want, trail)
    return best
