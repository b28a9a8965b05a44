"""Small Bizepel models for tests: configurations, random weights written as model folders."""
import numpy as np

from dafotar_util import write_model  # noqa: F401  (a folder with config.json and model.safetensors)


def dense(ff=48):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=24, groups=(3, 2), scale=1.7, shared_ff=40):
    ro = {"experts": experts, "top": top}
    if groups:
        ro["groups"] = {"count": groups[0], "keep": groups[1]}
    if scale is not None:
        ro["scale"] = scale
    return {"kind": "moe", "expert": {"ff": ff}, "router": ro, "shared": {"ff": shared_ff} if shared_ff else None}


def attention_layer(heads=4, kv_heads=2, dim=24, vdim=16, rot_dims=12, base=500.0, scale=None, window=21, keep=3, conv=4,
                    v_mix=True, mlp=None):
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5,
          "v_mix": v_mix}
    if conv:
        mx["conv"] = conv
    if rot_dims:
        mx["rot"] = {"base": base, "dims": rot_dims}
    if window:
        mx["mask"] = {"size": window, "keep_first": keep}
    return {"type": "attention", "mixer": mx, "mlp": mlp}


def scan_layer(inner=40, state=5, dt_rank=3, conv=4, mlp=None):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}, "mlp": mlp}


def delta_layer(heads=3, dim=12, rank=7, mlp=None):
    """``rank`` shapes the weights alone; the config does not name it."""
    return {"type": "general_delta", "mixer": {"heads": heads, "dim": dim}, "mlp": mlp, "_rank": rank}


def config(layers, vocab=96, width=32, eps=1e-5, taps=3, side=10, logit_scale=0.5):
    cfg = {"architecture": "Bizepel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if taps:
        cfg["canon"] = {"taps": taps}
    if side:
        cfg["token_side"] = {"dim": side}
    if logit_scale is not None:
        cfg["logit_scale"] = logit_scale
    return cfg


# Three configurations that differ in every size and option.  A: every kind of layer and both
# feed-forwards; values narrower than keys in sizes that no matrix-core kernel takes, part of a head
# rotated, windows that are no multiple of a page, a layer without v_mix between two with it, groups of
# experts.  B: sizes that the matrix-core kernels take (keys of 32 with values of 16, keys of 16
# with values of 32), as many key heads as query heads, a whole head rotated, no window on one layer,
# no kept tokens on another, no groups, one expert a token, no shared expert, a layer without feed-forward,
# no token input, no factor on the logits, heads of 32 in the recurrence.  C: a width that is no
# multiple of eight, one head everywhere, groups of one expert, every expert chosen, windows of 1 and
# 2, no rotation, convolutions of one and two taps, a side input of one channel, a factor above 1.
CFG_A = config([
    scan_layer(40, 5, 3, 4, mlp=dense(40)),
    attention_layer(heads=4, kv_heads=2, dim=24, vdim=16, rot_dims=12, base=500.0, window=21, keep=3, conv=4,
                    mlp=moe(6, 3, 24, (3, 2), 1.7, 40)),
    delta_layer(3, 12, 7, mlp=moe(4, 2, 16, (2, 1), 0.8, 24)),
    attention_layer(heads=2, kv_heads=1, dim=10, vdim=14, rot_dims=4, base=50.0, scale=0.4, window=13, keep=6, conv=3,
                    v_mix=False, mlp=dense(56)),
    attention_layer(heads=4, kv_heads=4, dim=20, vdim=8, rot_dims=20, base=90.0, window=9, keep=2, conv=2, mlp=dense(24)),
], vocab=150, width=48, eps=1e-5, taps=3, side=10, logit_scale=0.5)
CFG_B = config([
    attention_layer(heads=2, kv_heads=2, dim=32, vdim=16, rot_dims=32, base=2000.0, window=24, keep=5, conv=4,
                    mlp=moe(3, 1, 40, None, None, None)),
    delta_layer(2, 32, 16, mlp=None),
    attention_layer(heads=4, kv_heads=1, dim=16, vdim=32, rot_dims=8, base=100.0, window=None, conv=None, mlp=dense(64)),
    scan_layer(64, 16, 8, 2, mlp=dense(128)),
    attention_layer(heads=2, kv_heads=1, dim=64, vdim=32, rot_dims=16, base=40.0, window=17, keep=0, conv=5,
                    mlp=moe(4, 2, 32, (2, 2), 2.0, 64)),
], vocab=131, width=64, eps=1e-6, taps=4, side=None, logit_scale=None)
CFG_C = config([
    delta_layer(1, 10, 3, mlp=moe(4, 4, 12, (4, 4), 1.0, 12)),
    attention_layer(heads=1, kv_heads=1, dim=10, vdim=6, rot_dims=0, window=1, keep=0, conv=1, v_mix=False, mlp=None),
    scan_layer(9, 1, 1, 1, mlp=moe(5, 2, 20, (5, 3), 3.0, None)),
    attention_layer(heads=1, kv_heads=1, dim=12, vdim=20, rot_dims=2, base=10.0, window=2, keep=1, conv=2, mlp=dense(20)),
], vocab=64, width=36, eps=1e-6, taps=1, side=1, logit_scale=3.0)


def file_config(cfg):
    """The configuration as a config.json holds it."""
    out = dict(cfg)
    out["layers"] = [{k: v for k, v in l.items() if not k.startswith("_")} for l in cfg["layers"]]
    return out


def tensor_shapes(cfg, unused=False):
    """``unused``: with the first value-mixing layer's share, which a checkpoint may hold."""
    W = cfg["width"]
    side = (cfg.get("token_side") or {}).get("dim")
    taps = (cfg.get("canon") or {}).get("taps")
    out = {"embed": (cfg["vocab"], W), "embed.norm": (W,), "final.norm": (W,)}
    if side:
        out["side.embed"] = (cfg["vocab"], side * len(cfg["layers"]))
    mixed = False
    for i, l in enumerate(cfg["layers"]):
        p, mx, ml = f"l{i}.", l["mixer"], l["mlp"]
        for q in (1, 2) if ml else (1,):
            out[f"{p}norm{q}"] = (W,)
            out[f"{p}ls{q}"] = (W,)
            if taps:
                out[f"{p}canon{q}"] = (W, taps)
        m = p + "mix."
        if l["type"] == "attention":
            H, D, E = mx["heads"], mx["dim"], mx["vdim"]
            G = mx.get("kv_heads", H)
            for r, n in (("q", H * D), ("k", G * D), ("v", G * E)):
                out[m + r] = (n, W)
                out[f"{m}{r}.b"] = (n,)
                if mx.get("conv"):
                    out[f"{m}{r}.conv"] = (n, mx["conv"])
            out.update({m + "q.norm": (D,), m + "k.norm": (D,), m + "o": (W, H * E)})
            if mx["v_mix"]:
                if mixed or unused:
                    out[m + "vmix"] = ()
                mixed = True
        elif l["type"] == "mamba1":
            I, N, R = mx["inner"], mx["state"], mx["dt_rank"]
            out.update({m + "in": (2 * I, W), m + "conv": (I, mx["conv"]), m + "conv.b": (I,), m + "x": (R + 2 * N, I),
                        m + "dt": (I, R), m + "dt.b": (I,), m + "A_log": (I, N), m + "D": (I,), m + "o": (W, I)})
        else:
            C, R = mx["heads"] * mx["dim"], l["_rank"]
            out.update({m + n: (C, W) for n in ("r", "k", "v", "g", "a")})
            out.update({m + "a.b": (C,), m + "w1": (R, W), m + "w2": (C, R), m + "w0": (C,), m + "norm": (C,), m + "o": (W, C)})
        f = p + "mlp."
        if ml and ml["kind"] == "dense":
            out.update({f + "up": (ml["ff"], W), f + "down": (W, ml["ff"])})
        elif ml:
            E = ml["router"]["experts"]
            out.update({f + "router": (E, W), f + "correction": (E,)})
            for e in range(E):
                out.update({f"{f}e{e}.up": (ml["expert"]["ff"], W), f"{f}e{e}.down": (W, ml["expert"]["ff"])})
            if ml.get("shared"):
                ff = ml["shared"]["ff"]
                out.update({f + "shared.up": (ff, W), f + "shared.down": (W, ff)})
        if side:
            out.update({p + "side.gate": (side, W), p + "side.proj": (W, side), p + "side.norm": (W,)})
    return out


def random_weights(cfg, seed):
    """float32 arrays, already rounded to bfloat16 values so that either storage type holds the
    same numbers."""
    from zse_amd.weights.safetensors import bf16_bits_to_f32, f32_to_bf16_bits
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, unused=True).items():
        last = name.split(".")[-1]
        if name in ("embed", "side.embed"):
            a = rng.normal(0, 0.8, shape)
        elif last in ("norm", "norm1", "norm2"):
            a = 1.0 + rng.normal(0, 0.2, shape)
        elif last in ("ls1", "ls2"):
            a = rng.normal(0.8, 0.3, shape)
        elif last in ("canon1", "canon2"):
            a = rng.normal(0, 0.4, shape)
        elif last == "conv":
            a = rng.normal(0, 0.6, shape)
        elif last == "vmix":
            a = np.full(shape, 0.35 + 0.1 * rng.random())
        elif name.endswith("dt.b"):
            a = rng.normal(-1.0, 0.8, shape)
        elif last == "A_log":
            a = rng.normal(0.0, 0.7, shape)
        elif last in ("D", "w0"):
            a = rng.normal(0, 1.0, shape)
        elif last in ("b", "correction"):
            a = rng.normal(0, 0.3, shape)
        elif last == "router":
            a = rng.normal(0, 2.0 / np.sqrt(shape[-1]), shape)
        elif last == "up":
            a = rng.normal(0, 1.2 / np.sqrt(shape[-1]), shape)
        else:
            a = rng.normal(0, 1.0 / np.sqrt(shape[-1]), shape)
        out[name] = bf16_bits_to_f32(f32_to_bf16_bits(np.asarray(a, np.float32).reshape(-1))).reshape(shape)
    return out
