"""Small Fivitar and Fekulix configurations with random weights, for the tests of the hybrid decoders."""
from __future__ import annotations

import torch

YARN = {"factor": 8.0, "original": 64, "fast": 16.0, "slow": 2.0}


def lightning(heads, dim, vdim, decay=None):
    decay = decay or [round(1.0 - 0.5 ** (1 + 2 * i), 6) for i in range(heads)]
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}


def latent(heads, dim, rot, vdim, rank, base=1000.0, scaling=None, scale=None, dims=None):
    rot_cfg = {"base": base, "dims": dims or rot}
    if scaling:
        rot_cfg["scaling"] = scaling
    return {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "rot": rot_cfg,
            "scale": scale or (dim + rot) ** -0.5}


def delta(heads, kv_heads, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def grouped(heads, kv_heads, dim, vdim, rot, base=1000.0, scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5, "rot": {"base": base, "dims": rot}}


def gated_linear(heads, dim, vdim, tau):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}


def parallel(left, right, left_scale, right_scale):
    return {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}


def layer(kind, mixer, ff, weights_of=None):
    out = {"type": kind, "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}
    if weights_of is not None:
        out["weights_of"] = weights_of
    return out


def config_odd():
    """Sizes that are no multiple of a tile, a layer without feed-forward, every mixer running again, a chain of references."""
    d, a, l = delta(3, 3, 20, 36, 3), latent(3, 22, 10, 18, 30, base=500.0, scaling=YARN), lightning(5, 12, 28, [0.0, 0.4, 0.9, 0.999, 1.0])
    return {"architecture": "Fivitar", "vocab": 301, "width": 84, "norm": {"eps": 1e-4},
            "layers": [layer("delta", d, 100), layer("latent_attention", a, None), layer("lightning", l, 52),
                       layer("delta", d, 100, 0), layer("latent_attention", a, None, 1), layer("delta", d, 100, 3),
                       layer("lightning", l, 52, 2)]}


def config_wide():
    """Head sizes of real models, a few key heads shared by many value heads, two latent layers apart in every constant."""
    return {"architecture": "Fivitar", "vocab": 512, "width": 256, "norm": {"eps": 1e-6},
            "layers": [layer("latent_attention", latent(17, 64, 32, 128, 160, scaling=YARN), 320),
                       layer("delta", delta(4, 2, 128, 128, 4), 256),
                       layer("lightning", lightning(2, 128, 64), 192),
                       layer("latent_attention", latent(2, 128, 64, 48, 512, base=10000.0, scale=0.2), 320),
                       layer("delta", delta(2, 1, 64, 256, 1), None)]}


def config_tiny():
    """One head, one tap, one layer of a kind."""
    return {"architecture": "Fivitar", "vocab": 96, "width": 64, "norm": {"eps": 1e-5},
            "layers": [layer("lightning", lightning(1, 16, 16, [0.97]), 64), layer("delta", delta(1, 1, 16, 16, 1), 64),
                       layer("latent_attention", latent(1, 16, 8, 16, 16), 128)]}


def fekulix(vocab, width, eps, logit_scale, layers):
    return {"architecture": "Fekulix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale, "layers": layers}


def config_fek_odd():
    """Sizes that are no multiple of a tile, a layer without feed-forward, every mixer running again, a chain of references."""
    p = parallel(grouped(6, 2, 22, 18, 10, base=500.0, scale=0.3), gated_linear(3, 12, 28, 4.0), 0.9, 0.4)
    d = delta(4, 2, 20, 36, 3)
    return fekulix(301, 84, 1e-4, 0.7, [layer("channel_delta", d, 100), layer("parallel", p, None), layer("channel_delta", d, 100, 0),
                                        layer("parallel", p, None, 1), layer("channel_delta", d, 100, 2)])


def config_fek_wide():
    """Head sizes of real models, many query heads on one key head, parallel layers apart in every constant."""
    return fekulix(512, 256, 1e-6, 3.0,
                   [layer("parallel", parallel(grouped(18, 1, 128, 64, 128, base=1e5), gated_linear(2, 128, 128, 16.0), 0.5, 1.3), 320),
                    layer("channel_delta", delta(4, 1, 64, 128, 4), 256),
                    layer("parallel", parallel(grouped(4, 4, 64, 144, 48, scale=0.2), gated_linear(4, 32, 48, 1.0), 1.1, 0.25), 192),
                    layer("channel_delta", delta(2, 2, 128, 64, 6), None)])


def config_fek_tiny():
    """One head, one tap, constants of one."""
    return fekulix(96, 64, 1e-5, 1.0, [layer("parallel", parallel(grouped(1, 1, 16, 16, 2, scale=1.0), gated_linear(1, 16, 16, 1.0), 1.0, 1.0), 64),
                                       layer("channel_delta", delta(1, 1, 16, 16, 1), 128)])


CONFIGS = {"odd": config_odd, "wide": config_wide, "tiny": config_tiny, "fek_odd": config_fek_odd, "fek_wide": config_fek_wide,
           "fek_tiny": config_fek_tiny}


def ranks(m):
    """Of the low-rank maps of a mixer (only its tensors tell)."""
    return m["dim"] // 3 + 2, m["vdim"] // 4 + 1


def mixer_shapes(kind, m, width):
    if kind == "parallel":
        return {f"{side}.{n}": s for side, k in (("left", "grouped"), ("right", "gated_linear"))
                for n, s in mixer_shapes(k, m[side], width).items()}
    H, D, V = m["heads"], m["dim"], m["vdim"]
    if kind == "grouped":
        G = m["kv_heads"]
        s = {"q": (H * D, width), "k": (G * D, width), "v": (G * V, width), "o": (width, H * V)}
        if m.get("qk_norm", True):
            s.update({"q.norm": (D,), "k.norm": (D,)})
        return {**s, "g": (H, width)} if m.get("gated", True) else s
    if kind == "gated_linear":
        R = ranks(m)[0]
        return {"q": (H * D, width), "k": (H * D, width), "v": (H * V, width), "g": (H * V, width), "o": (width, H * V), "norm": (V,),
                "a1": (R, width), "a2": (H * D, R), "a2.b": (H * D,)}
    if kind == "latent_attention":
        R, C = m["rot_dim"], m["kv_rank"]
        return {"q": (H * (D + R), width), "dkv": (C + R, width), "dkv.norm": (C,), "uk": (H * D, C), "uv": (H * V, C), "sink": (H,),
                "o": (width, H * V)}
    if kind == "lightning":
        return {"q": (H * D, width), "k": (H * D, width), "v": (H * V, width), "g": (H * V, width), "norm": (H * V,), "o": (width, H * V)}
    G, n = m["kv_heads"], m["conv"]
    if kind == "channel_delta":
        R, S = ranks(m)
        return {"q": (G * D, width), "q.conv": (G * D, n), "k": (G * D, width), "k.conv": (G * D, n), "v": (H * V, width), "v.conv": (H * V, n),
                "b": (H, width), "A_log": (H,), "norm": (V,), "a1": (R, width), "a2": (H * D, R), "dt_bias": (H * D,), "g1": (S, width),
                "g2": (H * V, S), "o": (width, H * V)}
    return {"q": (G * D, width), "q.conv": (G * D, n), "k": (G * D, width), "k.conv": (G * D, n), "v": (H * V, width), "v.conv": (H * V, n),
            "b": (H, width), "a": (H, width), "A_log": (H,), "dt_bias": (H,), "norm": (V,), "g": (H * V, width), "o": (width, H * V)}


def shapes(cfg):
    d, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"]), "head": (cfg["vocab"], cfg["width"])}
    fek = cfg["architecture"] == "Fekulix"
    norm = lambda name: {name: (d,), name + ".b": (d,), name + ".alpha": ()} if fek else {name: (d,)}
    out.update(norm("final.norm"))
    for i, l in enumerate(cfg["layers"]):
        if "weights_of" in l:
            continue
        s = {"mix." + n: sh for n, sh in mixer_shapes(l["type"], l["mixer"], d).items()}
        s.update(norm("norm1"))
        if not fek:
            s.update({"rg1": (d, d), "rg1.b": (d,)})
        if l["mlp"] is not None:
            ff = l["mlp"]["ff"]
            s.update({"mlp.up": (ff, d), "mlp.down": (d, ff), **norm("norm2")})
            if not fek:
                s.update({"mlp.act": (2,), "rg2": (d, d), "rg2.b": (d,)})
        out.update({f"l{i}.{n}": sh for n, sh in s.items()})
    return out


def random_tensor(name, shape, g):
    t = torch.randn(shape, generator=g)
    if name.endswith(("A_log", "dt_bias")):
        t = t - 2.0                                        # decays between forgetting at once and keeping for long
    elif name.endswith("sink"):
        t = t + 1.0
    elif name.endswith("alpha"):
        t = 0.6 + 0.1 * t
    elif "norm" in name and name.endswith(".b"):
        t = 0.3 * t
    elif name.endswith("norm") or ".norm" in name:
        t = 1.0 + 0.3 * t
    elif name.endswith(".conv"):
        t = t * 0.7
    elif len(shape) == 2 and name != "embed":
        t = t * 1.5 / shape[1] ** 0.5
    return t.to(torch.bfloat16)


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    return {n: random_tensor(n, s, g) for n, s in shapes(cfg).items()}


def tokens(cfg, n, seed=1):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()
