"""Small Lurepel configurations and random weights for the tests: the tensor list is derived here from the configuration alone
(not from the package's manifest), the weights are drawn so that every mechanism moves the logits (norm weights away from one,
router scores that spread, corrections that change choices), and model folders are written with the package's safetensors
writer."""

from __future__ import annotations

import json
import os

import numpy as np
import torch


def rotation(dims, base, slowed=None):
    rot = {"base": base, "dims": dims}
    if slowed:
        rot["scaling"] = dict(zip(("factor", "low", "high", "original"), slowed))
    return rot


def attention(heads, kv_heads, dim, scale, chunk=0, dims=0, base=10000.0, slowed=None, mlp=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if chunk:
        mixer["mask"] = {"size": chunk}
    if dims:
        mixer["rot"] = rotation(dims, base, slowed)
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, identity=0):
    router = {"experts": experts, "top": top}
    if identity:
        router["identity"] = identity
    return {"kind": "moe", "router": router, "expert": {"ff": ff}}


SLOWED = (4.0, 1.0, 4.0, 64)
# All three feed-forwards; chunks a little longer than a page, every earlier key, and exactly a page; half a head turned with
# slowed pairs, a whole head without, no rotation; more identity experts than are used.
MIXED = {
    "architecture": "Lurepel", "vocab": 97, "width": 64, "norm": {"eps": 1e-5},
    "layers": [attention(4, 2, 32, 0.3, chunk=70, dims=16, base=500.0, slowed=SLOWED, mlp=moe(6, 3, 32, identity=2)),
               attention(3, 1, 16, 0.4, dims=16, base=500.0),
               attention(2, 2, 48, 0.25, chunk=64, mlp=dense(80)),
               attention(6, 3, 64, 0.2, chunk=33, dims=24, base=20000.0, slowed=(8.0, 0.5, 6.0, 32), mlp=moe(4, 1, 40, identity=3))],
}
# One head everywhere, every earlier key, one expert beside one that hands its input through, one of them used.
PLAIN = {
    "architecture": "Lurepel", "vocab": 131, "width": 96, "norm": {"eps": 1e-6},
    "layers": [attention(1, 1, 64, 0.2, dims=64, base=1000.0, mlp=moe(1, 1, 64, identity=1)),
               attention(1, 1, 32, 0.5, chunk=1, mlp=dense(128))],
}
# Sizes that are no multiples of 8; as many experts a row as there are; seventeen query heads to a key/value head; no identity.
ODD = {
    "architecture": "Lurepel", "vocab": 53, "width": 36, "norm": {"eps": 1e-3},
    "layers": [attention(5, 5, 12, 0.6, chunk=9, dims=6, base=50.0, mlp=moe(3, 3, 20)),
               attention(17, 1, 20, 0.4, dims=2, base=10.0, slowed=(16.0, 2.0, 2.0, 16), mlp=dense(50)),
               attention(2, 1, 6, 0.5, chunk=3, dims=4, base=300.0, mlp=moe(2, 4, 12, identity=2))],
}
# Wider heads: 96 and 80 (which is padded), 160, groups of eight, sixteen experts and five that hand their input through.
WIDE = {
    "architecture": "Lurepel", "vocab": 211, "width": 128, "norm": {"eps": 1e-6},
    "layers": [attention(8, 1, 96, 0.15, chunk=130, dims=96, base=250000.0, slowed=(16.0, 1.0, 4.0, 256), mlp=moe(16, 4, 64, identity=5)),
               attention(4, 4, 80, 0.2, dims=40, base=1000.0, mlp=dense(192)),
               attention(2, 1, 160, 0.1, chunk=200, dims=32, base=30000.0, slowed=(2.0, 1.0, 8.0, 128), mlp=moe(8, 2, 128, identity=1))],
}
CONFIGS = {"mixed": MIXED, "plain": PLAIN, "odd": ODD, "wide": WIDE}


def tensor_shapes(config):
    """{name: shape} of a configuration's checkpoint."""
    width = config["width"]
    shapes = {"embed": (config["vocab"], width), "embed.norm": (width,), "final.norm": (width,), "head": (config["vocab"], width)}

    def feed_forward(p, ff):
        shapes.update({p + "gate": (ff, width), p + "up": (ff, width), p + "down": (width, ff)})

    for index, layer in enumerate(config["layers"]):
        p, m, mlp = f"l{index}.", layer["mixer"], layer["mlp"]
        shapes[p + "norm1"] = (width,)
        shapes.update({p + "mix.q": (m["heads"] * m["dim"], width), p + "mix.k": (m["kv_heads"] * m["dim"], width), p + "mix.g": (m["heads"], width),
                       p + "mix.o": (width, m["heads"] * m["dim"])})
        if not mlp:
            continue
        shapes[p + "norm2"] = (width,)
        if mlp["kind"] == "dense":
            feed_forward(p + "mlp.", mlp["ff"])
            continue
        numbered = mlp["router"]["experts"] + mlp["router"].get("identity", 0)
        shapes.update({p + "mlp.router": (numbered, width), p + "mlp.correction": (numbered,)})
        for e in range(mlp["router"]["experts"]):
            feed_forward(f"{p}mlp.e{e}.", mlp["expert"]["ff"])
    return shapes


def bfloat(values):
    """float32 numbers that are exact in bfloat16."""
    return torch.from_numpy(np.asarray(values, np.float32)).to(torch.bfloat16).to(torch.float32).numpy()


def random_weights(config, seed, gain=1.0):
    """Matrices N(0, gain / sqrt(inputs)); router matrices twice that, so that scores spread; corrections N(0, 0.15), which change
    one choice in several; norm weights 1 + N(0, 0.3)."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in tensor_shapes(config).items():
        last = name.split(".")[-1]
        if name == "embed":
            values = rng.standard_normal(shape)
        elif last == "router":
            values = rng.standard_normal(shape) * 2.0 / np.sqrt(shape[1])
        elif last == "correction":
            values = rng.standard_normal(shape) * 0.15
        elif len(shape) == 2:
            values = rng.standard_normal(shape) * gain / np.sqrt(shape[1])
        else:
            values = 1.0 + 0.3 * rng.standard_normal(shape)
        out[name] = bfloat(values)
    return out


def write_model(folder, config, weights):
    from beholdd.weights import write_safetensors

    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as handle:
        json.dump(config, handle)
    write_safetensors(os.path.join(folder, "model.safetensors"),
                      {name: torch.from_numpy(np.ascontiguousarray(value)).to(torch.bfloat16) for name, value in weights.items()})
    return str(folder)


def drawn_config(seed):
    """A configuration whose every size, count, constant and layer order is drawn."""
    rng = np.random.default_rng(seed)
    pick = lambda *values: values[int(rng.integers(len(values)))]

    def feed_forward():
        kind = pick("none", "dense", "moe", "moe")
        if kind == "none":
            return None
        if kind == "dense":
            return dense(int(pick(36, 64, 100)))
        experts, identity = int(pick(1, 2, 5, 8)), int(pick(0, 1, 2, 4))
        return moe(experts, int(rng.integers(1, min(experts + identity, 4) + 1)), int(pick(8, 20, 32, 64)), identity)

    layers = []
    for _ in range(int(rng.integers(1, 5))):
        kv_heads, dim = int(pick(1, 2, 3)), int(pick(8, 12, 32, 64, 96))
        dims = int(pick(0, *[d for d in (2, 8, 12, 32, 64, 96) if d <= dim]))
        slowed = pick(None, (float(pick(2.0, 6.0, 32.0)), float(pick(0.5, 1.0)), float(pick(2.0, 4.0)), int(pick(16, 64, 256))))
        layers.append(attention(kv_heads * int(pick(1, 2, 4, 8)), kv_heads, dim, float(pick(0.1, 0.2, 0.4)), chunk=int(pick(0, 1, 3, 64, 65, 100)),
                                dims=dims, base=float(pick(100.0, 10000.0, 1e6)), slowed=slowed if dims else None, mlp=feed_forward()))
    return {"architecture": "Lurepel", "vocab": int(pick(37, 64, 150, 301)), "width": int(pick(24, 40, 52, 64, 72, 96, 130)),
            "norm": {"eps": float(pick(1e-6, 1e-5, 1e-3))}, "layers": layers}
