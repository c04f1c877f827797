"""Small random models for the tests of stacks of attention / linear-attention layers: configurations as config.json has
them, weights rounded to bf16, as the product's tensor source and as float64 arrays for the plain statement."""
import numpy as np


def bf16_bits(x):
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def bf16_values(bits):
    return (bits.astype(np.uint32) << 16).view(np.float32)


def rounded(x):
    """x to the nearest bf16, as float64."""
    return bf16_values(bf16_bits(x)).astype(np.float64)


def attention(heads, kv_heads, dim, vdim, scale=None, diff=0.2, mlp=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale, "diff": diff}}


def lightning(heads, dim, vdim, decay=None, mlp=None):
    decay = list(np.linspace(0.5, 0.995, heads)) if decay is None else decay
    return {"type": "lightning", "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def config(vocab, width, layers, loop=None, eps=1e-5):
    return {"architecture": "Komirax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers, "loop": loop}


# ---- Vifivik -------------------------------------------------------------------------------------------------------------
def latent(heads, dim, rot, vdim, rank, scale=None, base=10000.0, kv_from=None, ff=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "rot": {"base": base, "dims": rot},
         "scale": (dim + rot) ** -0.5 if scale is None else scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": ff and dense(ff)}


def retention(heads, dim, vdim, decay=None, ff=None):
    decay = list(1.0 - 2.0 ** -np.linspace(2, 9, heads)) if decay is None else decay
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, "mlp": ff and dense(ff)}


def mamba2(heads, vdim, state, groups=1, conv=4, norm_groups=1, ff=None):
    return {"type": "mamba2", "mlp": ff and dense(ff), "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
                                                                 "conv": conv, "norm_groups": norm_groups}}


def vifivik(vocab, width, layers, eps=1e-5, cap=20.0):
    return {"architecture": "Vifivik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers, "logit_softcap": cap}


def vifivik_weights(cfg, seed):
    """name -> bf16 bits.  Queries and latents are large enough for the softmax to have favourites; sinks, step biases and decay
    rates differ from head to head."""
    g = np.random.default_rng(seed)
    w, v, t = cfg["width"], cfg["vocab"], {}

    def mat(name, rows, cols, scale=1.0):
        t[name] = g.standard_normal((rows, cols)) * (scale / np.sqrt(cols))

    def norm(name, n, mean=1.0):
        t[name] = mean + 0.1 * g.standard_normal(n)
    t["embed"] = g.standard_normal((v, w))
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", l["mixer"]
        norm(f"l{i}.norm1", w, 0.5)
        if l["type"] == "latent_attention":
            H, d, e, r = m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
            mat(p + "q", H * (d + e), w, 1.5)
            if "kv_from" not in m:
                mat(p + "dkv", r + e, w)
                norm(p + "dkv.norm", r)
            mat(p + "uk", H * d, r)
            mat(p + "uv", H * m["vdim"], r)
            t[p + "sink"] = 1.5 * g.standard_normal(H)
            mat(p + "g", H, w)
            mat(p + "o", w, H * m["vdim"])
        elif l["type"] == "retention":
            nk, nv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            for n, c in (("q", nk), ("k", nk), ("v", nv), ("g", nv)):
                mat(p + n, c, w)
            mat(p + "o", w, nv)
        else:
            inner, ch, H = m["heads"] * m["vdim"], m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"], m["heads"]
            mat(p + "in", inner + ch + H, w)
            mat(p + "conv", ch, m["conv"], 1.5)
            t[p + "conv.b"] = 0.2 * g.standard_normal(ch)
            t[p + "dt_bias"] = np.linspace(-5.0, -0.5, H) if H > 1 else np.array([-3.0])
            t[p + "A_log"] = np.linspace(2.0, -1.0, H) if H > 1 else np.array([0.5])
            t[p + "D"] = g.standard_normal(H)
            norm(p + "norm", inner)
            mat(p + "o", w, inner)
        if l["mlp"]:
            norm(f"l{i}.norm2", w, 0.5)
            ff = l["mlp"]["ff"]
            mat(f"l{i}.mlp.gate", ff, w)
            mat(f"l{i}.mlp.up", ff, w)
            mat(f"l{i}.mlp.down", w, ff)
    norm("final.norm", w)
    mat("head", v, w, 4.0)
    return {n: bf16_bits(x) for n, x in t.items()}


def weights(cfg, seed):
    """name -> bf16 bits.  Output projections are scaled down and the embeddings carry evenly spaced components along the
    routers' (orthonormal) directions, so that no routing decision is a close call and bf16 runs pick the same experts."""
    if cfg["architecture"] == "Vifivik":
        return vifivik_weights(cfg, seed)
    g = np.random.default_rng(seed)
    w, v = cfg["width"], cfg["vocab"]
    t = {}

    def mat(name, rows, cols, scale=1.0):
        t[name] = g.standard_normal((rows, cols)) * (scale / np.sqrt(cols))

    def norm(name, n):
        t[name] = 1.0 + 0.1 * g.standard_normal(n)
    most = max([l["mlp"]["router"]["experts"] for l in cfg["layers"] if l["mlp"] and l["mlp"]["kind"] == "moe"] or [0])
    assert most <= w
    dirs = np.linalg.qr(g.standard_normal((w, w)))[0][:most] if most else np.zeros((0, w))
    t["embed"] = 0.5 * g.standard_normal((v, w))
    if most:
        t["embed"] -= (t["embed"] @ dirs.T) @ dirs
        gap = np.sqrt(w) * 2.0 / most
        t["embed"] += np.stack([g.permutation(most) - (most - 1) / 2 for _ in range(v)]) * gap @ dirs
    for i, l in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", l["mixer"], l["mlp"]
        norm(p + "norm1", w)
        if l["type"] == "attention":
            for n, c in (("q", m["heads"] * 2 * m["dim"]), ("k", m["kv_heads"] * 2 * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                mat(p + "mix." + n, c, w)
                t[p + f"mix.{n}.b"] = 0.3 * g.standard_normal(c)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                t[p + "mix." + n] = 0.8 / np.sqrt(m["dim"]) * g.standard_normal(m["dim"])
            mat(p + "mix.o", w, m["heads"] * m["vdim"], 0.4)
        else:
            nk, nv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            for n, c in (("q", nk), ("k", nk), ("v", nv), ("g", nv)):
                mat(p + "mix." + n, c, w)
            mat(p + "mix.o", w, nv, 0.4)
            norm(p + "mix.norm", nv)
        if f is None:
            continue
        norm(p + "norm2", w)
        if f["kind"] == "dense":
            mat(p + "mlp.up", f["ff"], w)
            mat(p + "mlp.down", w, f["ff"], 0.6)
        else:
            e, ff = f["router"]["experts"], f["expert"]["ff"]
            t[p + "mlp.router"] = dirs[g.permutation(most)[:e]] * 1.5
            for j in range(e):
                mat(p + f"mlp.e{j}.up", ff, w)
                mat(p + f"mlp.e{j}.down", w, ff, 0.3)
    norm("final.norm", w)
    mat("head", v, w, 2.0)
    return {n: bf16_bits(x) for n, x in t.items()}


def plain_weights(tensors):
    return {n: bf16_values(x).astype(np.float64) for n, x in tensors.items()}


class Tensors:
    """What a loader needs of a weight file, over arrays in memory."""

    def __init__(self, tensors):
        self.t = tensors

    def bf16(self, name, shape=None):
        assert shape is None or self.t[name].shape == tuple(shape), name
        return self.t[name]

    def f32(self, name, shape=None):
        return bf16_values(self.bf16(name, shape))
