"""Tiny Pemalorn configurations for the tests.  They differ from each other in every size, in the order of the layers
and in what they have at all: a loop in the middle, over the whole model, of one pass, or none; convolutions of one,
two, three and five taps or none; a token table or none; windows shorter than, equal to and longer than a cache page, of
one token, or none; rotations of a whole head, of part of it or of nothing, stretched or not; grouped, single and
ungrouped key heads; values of another size than keys; routers with many, some and no identity experts, one expert
chosen, all chosen; layers without a feed-forward."""
from tiny_nelutar import write_model as _write


def tiny_s():
    """Five layers, the middle two twice (seven runs): latent attention (window 20, shorter than a page; 3 heads, a
    stretched rotation of 8), attention (6 heads on 2, 8 of 24 features rotate, values of 40), latent attention with
    other sizes and a window of 70 without a feed-forward, attention of one head, latent attention that sees all."""
    return {
        "architecture": "Pemalorn", "vocab": 211, "width": 96, "norm": {"eps": 1e-5}, "canon": {"taps": 3},
        "token_side": {"dim": 12}, "loop": {"start": 1, "stop": 3, "times": 2},
        "layers": [
            {"type": "latent_attention", "mixer": {
                "heads": 3, "dim": 24, "rot_dim": 8, "vdim": 40, "q_rank": 48, "kv_rank": 56, "scale": 0.21,
                "rot": {"base": 500.0, "dims": 8, "scaling": {"factor": 4.0, "original": 64, "fast": 16.0, "slow": 1.0}},
                "mask": {"size": 20}},
             "mlp": {"kind": "moe", "expert": {"ff": 40}, "router": {"experts": 6, "identity": 3, "top": 3}}},
            {"type": "attention", "mixer": {"heads": 6, "kv_heads": 2, "dim": 24, "vdim": 40, "scale": 0.3,
                                            "rot": {"base": 5000.0, "dims": 8}},
             "mlp": {"kind": "moe", "expert": {"ff": 24}, "router": {"experts": 4, "identity": 1, "top": 2}}},
            {"type": "latent_attention", "mixer": {
                "heads": 5, "dim": 16, "rot_dim": 16, "vdim": 24, "q_rank": 32, "kv_rank": 40, "scale": 0.3,
                "rot": {"base": 10000.0, "dims": 16}, "mask": {"size": 70}},
             "mlp": None},
            {"type": "attention", "mixer": {"heads": 1, "kv_heads": 1, "dim": 32, "vdim": 16, "scale": 0.2,
                                            "rot": {"base": 100.0, "dims": 32}},
             "mlp": {"kind": "moe", "expert": {"ff": 16}, "router": {"experts": 3, "identity": 5, "top": 4}}},
            {"type": "latent_attention", "mixer": {
                "heads": 2, "dim": 32, "rot_dim": 8, "vdim": 32, "q_rank": 24, "kv_rank": 64, "scale": 0.18,
                "rot": {"base": 1000.0, "dims": 8, "scaling": {"factor": 3.0, "original": 500, "fast": 20.0, "slow": 0.7}}},
             "mlp": {"kind": "moe", "expert": {"ff": 32}, "router": {"experts": 8, "identity": 2, "top": 1}}},
        ],
    }


def tiny_t():
    """Sizes that suit no vector access and no matrix-core tile: a width of 100, heads of 20,
    ranks of 36 and 27, values of 10, two taps, a token table of 5 numbers a layer, one pass over the last layer; a
    router without identity experts that chooses all, one whose identity experts are most of it."""
    return {
        "architecture": "Pemalorn", "vocab": 77, "width": 100, "norm": {"eps": 1e-6}, "canon": {"taps": 2},
        "token_side": {"dim": 5}, "loop": {"start": 2, "stop": 3, "times": 1},
        "layers": [
            {"type": "attention", "mixer": {"heads": 3, "kv_heads": 3, "dim": 20, "vdim": 10, "scale": 0.5,
                                            "rot": {"base": 70.0, "dims": 0}},
             "mlp": {"kind": "moe", "expert": {"ff": 28}, "router": {"experts": 5, "top": 5}}},
            {"type": "latent_attention", "mixer": {
                "heads": 4, "dim": 20, "rot_dim": 4, "vdim": 12, "q_rank": 27, "kv_rank": 36, "scale": 0.35,
                "rot": {"base": 60.0, "dims": 4}, "mask": {"size": 33}},
             "mlp": {"kind": "moe", "expert": {"ff": 20}, "router": {"experts": 2, "identity": 9, "top": 3}}},
            {"type": "attention", "mixer": {"heads": 5, "kv_heads": 1, "dim": 12, "vdim": 22, "scale": 0.4,
                                            "rot": {"base": 1000.0, "dims": 6}},
             "mlp": None},
        ],
    }


def tiny_u():
    """The whole model three times (loop from the first layer to the last), five taps; a window of one token (a query
    sees itself and the sink only), a window of exactly a page, and one of 64 experts; no identity experts in one
    layer, as many as experts in another."""
    return {
        "architecture": "Pemalorn", "vocab": 130, "width": 64, "norm": {"eps": 1e-5}, "canon": {"taps": 5},
        "token_side": {"dim": 16}, "loop": {"start": 0, "stop": 3, "times": 3},
        "layers": [
            {"type": "latent_attention", "mixer": {
                "heads": 4, "dim": 8, "rot_dim": 2, "vdim": 8, "q_rank": 16, "kv_rank": 16, "scale": 1.0,
                "rot": {"base": 20.0, "dims": 2}, "mask": {"size": 1}},
             "mlp": {"kind": "moe", "expert": {"ff": 16}, "router": {"experts": 64, "identity": 64, "top": 6}}},
            {"type": "attention", "mixer": {"heads": 4, "kv_heads": 1, "dim": 16, "vdim": 64, "scale": 0.5,
                                            "rot": {"base": 200.0, "dims": 16}},
             "mlp": {"kind": "moe", "expert": {"ff": 8}, "router": {"experts": 4, "top": 2}}},
            {"type": "latent_attention", "mixer": {
                "heads": 8, "dim": 16, "rot_dim": 8, "vdim": 16, "q_rank": 64, "kv_rank": 32, "scale": 0.25,
                "rot": {"base": 300.0, "dims": 8, "scaling": {"factor": 8.0, "original": 32, "fast": 4.0, "slow": 1.0}},
                "mask": {"size": 64}},
             "mlp": {"kind": "moe", "expert": {"ff": 24}, "router": {"experts": 4, "identity": 4, "top": 2}}},
        ],
    }


def tiny_v():
    """Nothing optional: no loop, no convolutions, no token table, no window, no stretch."""
    return {
        "architecture": "Pemalorn", "vocab": 90, "width": 48, "norm": {"eps": 1e-5},
        "layers": [
            {"type": "latent_attention", "mixer": {
                "heads": 2, "dim": 16, "rot_dim": 8, "vdim": 24, "q_rank": 24, "kv_rank": 32, "scale": 0.3,
                "rot": {"base": 400.0, "dims": 8}},
             "mlp": {"kind": "moe", "expert": {"ff": 16}, "router": {"experts": 4, "identity": 2, "top": 2}}},
            {"type": "attention", "mixer": {"heads": 2, "kv_heads": 2, "dim": 16, "vdim": 16, "scale": 0.3,
                                            "rot": {"base": 400.0, "dims": 4}},
             "mlp": None},
        ],
    }


def medium_n():
    """Sizes of a real model's kind, so that the kernels for aligned sizes run (matrix-core attention with heads of 128
    and latents of 512, strip and skinny products, the library's product, experts on the matrix cores): width 1,024."""
    moe = {"kind": "moe", "expert": {"ff": 512}, "router": {"experts": 8, "identity": 2, "top": 2}}
    return {
        "architecture": "Pemalorn", "vocab": 1000, "width": 1024, "norm": {"eps": 1e-6}, "canon": {"taps": 4},
        "token_side": {"dim": 128}, "loop": {"start": 0, "stop": 2, "times": 2},
        "layers": [
            {"type": "latent_attention", "mixer": {
                "heads": 8, "dim": 128, "rot_dim": 64, "vdim": 128, "q_rank": 384, "kv_rank": 512, "scale": 192 ** -0.5,
                "rot": {"base": 10000.0, "dims": 64, "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}},
                "mask": {"size": 256}}, "mlp": moe},
            {"type": "attention", "mixer": {"heads": 8, "kv_heads": 2, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                                            "rot": {"base": 500000.0, "dims": 64}}, "mlp": moe},
        ],
    }


def write_model(raw, out_dir, seed, std=0.08, norm_std=0.1, router_gain=6.0):
    """A model folder with random weights through the package's own writer (tiny_nelutar.write_model)."""
    return _write(raw, out_dir, seed, std=std, norm_std=norm_std, router_gain=router_gain)
