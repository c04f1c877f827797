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


def weights(cfg, seed):
    """name -> bf16 bits.  Output projections are scaled down and the embeddings carry evenly spaced components along the
    routers' (orthonormal) directions, so that no routing decision is a close call and bf16 runs pick the same experts."""
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
