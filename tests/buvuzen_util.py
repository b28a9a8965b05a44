"""Small Buvuzen models for tests: configurations, random weights written as model folders."""
import copy

import numpy as np

from dafotar_util import write_model  # noqa: F401  (a folder with config.json and model.safetensors)


def moe(experts=5, top=2, ff=24, shared_ff=40, identity=1, scale=1.6, groups=(2, 1)):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "identity": identity, "scale": scale},
         "shared": {"ff": shared_ff} if shared_ff else None}
    if groups is not None:
        m["router"]["groups"] = dict(zip(("count", "keep"), groups))
    return m


def layer(heads=4, kv_heads=2, dim=24, vdim=None, scale=None, window=20, mlp=None):
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim or dim, "scale": scale if scale is not None else dim ** -0.5}
    if window:
        mx["mask"] = {"size": window}
    return {"type": "attention", "mixer": mx, "mlp": mlp}


def again(layers, *orders):
    """The layers, then for each number in ``orders`` another layer with that one's weights."""
    return layers + [dict(copy.deepcopy(layers[j]), weights_of=j) for j in orders]


def config(layers, vocab=96, width=32, eps=1e-5, scale=5.3, logit_scale=0.7):
    return {"architecture": "Buvuzen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "logit_scale": logit_scale, "layers": layers}


# Three configurations that differ in every size and option.  A: heads that no matrix-core attention
# kernel takes, values narrower and wider than keys, shared and unshared key heads, three groups of
# which two stay, identity experts, a layer without feed-forward, one without a window, weights used
# again across another layer.  B: sizes that the matrix-core kernels take (heads of 64 and 32, values half
# and twice as wide, width 64), one group, no shared expert in one layer, no identity experts there.
# C: a width that is no multiple of eight, one head, every expert chosen, windows 1 and 2, groups of one
# expert each, the first layer with the weights of the third one, numbers of 1.
CFG_A = config(again([layer(heads=6, kv_heads=2, dim=24, vdim=20, window=13, mlp=moe(7, 3, 24, 40, identity=2, scale=2.2, groups=(3, 2))),
                      layer(heads=3, kv_heads=3, dim=20, vdim=28, scale=0.4, window=29, mlp=None),
                      layer(heads=4, kv_heads=1, dim=12, vdim=12, window=None, mlp=moe(3, 1, 16, 24, identity=1, scale=0.8, groups=None))],
                     0, 1, 0), vocab=200, width=48, eps=1e-5, scale=5.3, logit_scale=0.7)
CFG_B = config(again([layer(heads=4, kv_heads=2, dim=64, vdim=32, window=24, mlp=moe(5, 2, 40, 56, identity=3, scale=3.0, groups=(2, 1))),
                      layer(heads=3, kv_heads=1, dim=32, vdim=64, scale=0.3, window=37, mlp=moe(4, 2, 32, None, identity=0, scale=1.0, groups=(1, 1)))],
                     1, 0), vocab=131, width=64, eps=1e-6, scale=1.7, logit_scale=2.5)
CFG_C = config([dict(layer(heads=1, kv_heads=1, dim=10, vdim=6, window=2, mlp=moe(2, 4, 12, 12, identity=2, scale=1.0, groups=(4, 4))), weights_of=2),
                layer(heads=1, kv_heads=1, dim=16, vdim=16, scale=1.0, window=1, mlp=moe(3, 1, 20, 8, identity=1, scale=1.0, groups=(4, 2))),
                layer(heads=1, kv_heads=1, dim=10, vdim=6, window=2, mlp=moe(2, 4, 12, 12, identity=2, scale=1.0, groups=(4, 4)))],
               vocab=64, width=36, eps=1e-6, scale=1.0, logit_scale=1.0)


def tensor_shapes(cfg):
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "head": (cfg["vocab"], W), "final.norm": (W,)}
    for i, l in enumerate(cfg["layers"]):
        if l.get("weights_of") is not None:
            continue
        p, mx = f"l{i}.", l["mixer"]
        H, G, D, E = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
        m = p + "mix."
        out.update({p + "norm1": (W,), m + "q": (H * D, W), m + "k": (G * D, W), m + "v": (G * E, W), m + "q.norm": (D,),
                    m + "k.norm": (D,), m + "sink": (H,), m + "g": (H, W), m + "o": (W, H * E)})
        ml, f = l["mlp"], p + "mlp."
        if not ml:
            continue
        n, ff = ml["router"]["experts"] + ml["router"]["identity"], ml["expert"]["ff"]
        out.update({p + "norm2": (W,), f + "router": (n, W), f + "correction": (n,)})
        for e in range(ml["router"]["experts"]):
            out.update({f"{f}e{e}.gate": (ff, W), f"{f}e{e}.up": (ff, W), f"{f}e{e}.down": (W, ff)})
        if ml.get("shared"):
            ff = ml["shared"]["ff"]
            out.update({f + "shared.gate": (ff, W), f + "shared.up": (ff, W), f + "shared.down": (W, ff), f + "shared.sg": (1, W)})
    return out


def random_weights(cfg, seed):
    """float32 arrays, already rounded to bfloat16 values so that either storage type holds the
    same numbers.  Projections that read the stream are drawn for a stream of unit size (the stream
    itself is as large as the embedding's scale makes it, so routers are drawn narrower)."""
    from zse_amd.weights.safetensors import bf16_bits_to_f32, f32_to_bf16_bits
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.split(".")[-1]
        if name == "embed":
            a = rng.normal(0, 0.7, shape)
        elif name.endswith("q.norm") or name.endswith("k.norm"):
            a = 1.0 + rng.normal(0, 0.2, shape)
        elif last in ("norm1", "norm2", "norm"):
            a = rng.normal(0, 0.3, shape)
        elif last == "sink":
            a = rng.normal(0.5, 1.5, shape)
        elif last == "correction":
            a = rng.normal(-0.1, 0.2, shape)
        elif last == "router":
            a = rng.normal(0, 0.8 / np.sqrt(shape[-1]), shape)
        elif last in ("g", "sg"):
            a = rng.normal(0, 0.5 / np.sqrt(shape[-1]), shape)
        else:
            a = rng.normal(0, 1.0 / np.sqrt(shape[-1]), shape)
        out[name] = bf16_bits_to_f32(f32_to_bf16_bits(a.astype(np.float32)))
    return out
