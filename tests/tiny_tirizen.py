"""Tiny Tirizen configurations for the tests.  They differ from each other in every size, in the order of the layers and
in what they have at all: one, two, three and five streams; layers that read the keys of the layer before, of one far
back, or none; grouped, single and ungrouped key heads; values of another size than keys; temperatures that grow every
token, at page borders, never; decays of several ranks and exponents; key sizes below and above what a wavefront's lanes
hold in one piece; dense feed-forwards, mixtures in which one expert, some or all are chosen, and none."""
from tiny_nelutar import write_model as _write


def tiny_a():
    """Five layers, three streams: attention, gla, attention that reads the first one's keys across the gla, attention
    without a feed-forward and with other sizes, attention that reads that one's keys."""
    return {
        "architecture": "Tirizen", "vocab": 203, "width": 96, "norm": {"eps": 1e-5}, "embedding": {"scale": 7.0},
        "max_positions": 1500, "residual_mult": 0.6, "streams": 3, "logit_scale": 0.4,
        "layers": [
            {"type": "attention", "mixer": {"heads": 6, "kv_heads": 3, "dim": 24, "vdim": 40, "scale": 0.25,
                                            "q_temp": {"coef": 0.4, "every": 20}},
             "mlp": {"kind": "moe", "expert": {"ff": 40}, "router": {"experts": 6, "top": 3}}},
            {"type": "gla", "mixer": {"heads": 3, "dim": 20, "vdim": 36, "tau": 8.0},
             "mlp": {"kind": "dense", "ff": 112}},
            {"type": "attention", "mixer": {"heads": 6, "kv_heads": 3, "dim": 24, "vdim": 40, "scale": 0.3, "kv_from": 0,
                                            "q_temp": {"coef": 0.9, "every": 64}},
             "mlp": {"kind": "moe", "expert": {"ff": 24}, "router": {"experts": 4, "top": 1}}},
            {"type": "attention", "mixer": {"heads": 4, "kv_heads": 1, "dim": 32, "vdim": 16, "scale": 0.2,
                                            "q_temp": {"coef": 0.1, "every": 1}},
             "mlp": None},
            {"type": "attention", "mixer": {"heads": 8, "kv_heads": 1, "dim": 32, "vdim": 16, "scale": 0.15, "kv_from": 3},
             "mlp": {"kind": "dense", "ff": 64}},
        ],
    }


def tiny_b():
    """Sizes that suit no vector access and no matrix-core tile: a width of 100, key sizes of 20 and 13, values of 10 and
    7, five streams; all experts chosen; a gla layer without a feed-forward, a decay that is sigmoid itself."""
    return {
        "architecture": "Tirizen", "vocab": 77, "width": 100, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
        "max_positions": 300, "residual_mult": 1.0, "streams": 5, "logit_scale": 1.0,
        "layers": [
            {"type": "gla", "mixer": {"heads": 5, "dim": 13, "vdim": 7, "tau": 1.0}, "mlp": None},
            {"type": "attention", "mixer": {"heads": 3, "kv_heads": 3, "dim": 20, "vdim": 10, "scale": 0.5,
                                            "q_temp": {"coef": 0.25, "every": 33}},
             "mlp": {"kind": "moe", "expert": {"ff": 28}, "router": {"experts": 5, "top": 5}}},
            {"type": "attention", "mixer": {"heads": 3, "kv_heads": 3, "dim": 20, "vdim": 10, "scale": 0.4, "kv_from": 1,
                                            "q_temp": {"coef": 0.25, "every": 33}},
             "mlp": {"kind": "moe", "expert": {"ff": 20}, "router": {"experts": 11, "top": 2}}},
            {"type": "gla", "mixer": {"heads": 2, "dim": 70, "vdim": 30, "tau": 24.0}, "mlp": {"kind": "dense", "ff": 60}},
        ],
    }


def tiny_c():
    """gla layers only but one, two streams: a key size of 128 and of 200 (a column's state in several pieces), one head,
    one value; 40 experts."""
    return {
        "architecture": "Tirizen", "vocab": 130, "width": 64, "norm": {"eps": 1e-5}, "embedding": {"scale": 3.5},
        "max_positions": 2048, "residual_mult": 0.35, "streams": 2, "logit_scale": 2.0,
        "layers": [
            {"type": "gla", "mixer": {"heads": 2, "dim": 128, "vdim": 48, "tau": 16.0},
             "mlp": {"kind": "moe", "expert": {"ff": 16}, "router": {"experts": 40, "top": 6}}},
            {"type": "gla", "mixer": {"heads": 1, "dim": 200, "vdim": 1, "tau": 4.0}, "mlp": {"kind": "dense", "ff": 72}},
            {"type": "attention", "mixer": {"heads": 2, "kv_heads": 2, "dim": 16, "vdim": 64, "scale": 0.5}, "mlp": None},
            {"type": "gla", "mixer": {"heads": 4, "dim": 8, "vdim": 24, "tau": 2.5},
             "mlp": {"kind": "moe", "expert": {"ff": 8}, "router": {"experts": 2, "top": 1}}},
        ],
    }


def tiny_d():
    """One stream and one layer of each kind; every optional key left out."""
    return {
        "architecture": "Tirizen", "vocab": 90, "width": 48, "norm": {"eps": 1e-5}, "max_positions": 256,
        "layers": [
            {"type": "attention", "mixer": {"heads": 2, "dim": 16, "scale": 0.3}, "mlp": {"kind": "dense", "ff": 40}},
            {"type": "gla", "mixer": {"heads": 2, "dim": 16, "tau": 10.0}, "mlp": None},
        ],
    }


def medium():
    """Sizes of a real model's kind, so that the kernels for aligned sizes run (matrix-core attention with heads of 128,
    strip and skinny products, the library's product, experts on the matrix cores, segments of the scan): width 1,024."""
    moe = {"kind": "moe", "expert": {"ff": 512}, "router": {"experts": 8, "top": 2}}
    att = {"heads": 8, "kv_heads": 2, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "q_temp": {"coef": 0.2, "every": 100}}
    return {
        "architecture": "Tirizen", "vocab": 1000, "width": 1024, "norm": {"eps": 1e-6}, "embedding": {"scale": 12.0},
        "max_positions": 1024, "residual_mult": 0.8, "streams": 4, "logit_scale": 0.5,
        "layers": [
            {"type": "gla", "mixer": {"heads": 4, "dim": 128, "vdim": 256, "tau": 16.0}, "mlp": moe},
            {"type": "attention", "mixer": att, "mlp": {"kind": "dense", "ff": 2048}},
            {"type": "attention", "mixer": dict(att, kv_from=1), "mlp": moe},
        ],
    }


def with_defaults(raw):
    """The configuration with every optional key written out, as the plain implementation reads it."""
    raw = {"embedding": {"scale": 1.0}, "residual_mult": 1.0, "streams": 1, "logit_scale": 1.0, **raw}
    layers = []
    for layer in raw["layers"]:
        m = dict(layer["mixer"])
        m.setdefault("vdim", m["dim"])
        if layer["type"] == "attention":
            m.setdefault("kv_heads", m["heads"])
        layers.append(dict(layer, mixer=m))
    return dict(raw, layers=layers)


def write_model(raw, out_dir, seed, std=0.08, norm_std=0.1, router_gain=6.0):
    """A model folder with random weights through the package's own writer (tiny_nelutar.write_model)."""
    return _write(raw, out_dir, seed, std=std, norm_std=norm_std, router_gain=router_gain)
