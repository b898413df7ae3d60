"""Small configurations of the Koketar design for the tests, with random weights and the float64 restatement of
oracle/parallel_model.py."""
from oracle import parallel_model


def window(heads=6, kv_heads=2, dim=24, vdim=40, size=21, scale=0.3, rotated=14, base=5000.0, factor=3.0):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": size},
            "rot": {"base": base, "dims": rotated, "scaling": {"factor": factor}}}


def delta(heads=4, kv_heads=2, dim=20, vdim=28, conv=4):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def dense(ff=104, limit=0.9):
    return {"kind": "dense", "ff": ff, "limit": limit}


def parallel(left=None, right=None, left_scale=0.8, right_scale=0.45, mlp=None):
    return {"type": "parallel", "mlp": mlp,
            "mixer": {"left": left or window(), "right": right or delta(), "left_scale": left_scale,
                      "right_scale": right_scale}}


def config(*layers, vocab=90, width=72, eps=1e-5, mult=0.7, softcap=12.0):
    return {"architecture": "Koketar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
            "logit_softcap": softcap, "layers": list(layers)}


def expected_logits(cfg, weights, tokens):
    return parallel_model.forward(cfg, weights, tokens)[0]
