"""Small layered-decoder configurations and comparisons for the tests: random weights, the float64
restatement of oracle/hybrid_model.py, errors relative to the expected values' root mean square."""
import numpy as np

from llmopt_amd.layered_model import LayeredConfig, LayeredModel
from llmopt_amd.safetensors_file import from_bfloat16, to_bfloat16
from oracle import hybrid_model



def attention(heads=6, kv_heads=3, dim=24, vdim=40, chunk=20, scale=0.3, softcap=8.0, v_mix=True, mlp=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                      "softcap": softcap, "v_mix": v_mix, "mask": {"size": chunk}}}


def mamba2(heads=6, vdim=20, state=24, groups=2, conv=4, norm_groups=3, mlp=None):
    return {"type": "mamba2", "mlp": mlp,
            "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                      "norm_groups": norm_groups}}


def dense(ff=112):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=40, shared=56):
    f = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    if shared:
        f["shared"] = {"ff": shared}
    return f


def config(*layers, vocab=90, width=72, eps=1e-5, scale=1.5):
    return {"architecture": "Barovik", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "layers": list(layers)}


def make_weights(cfg, seed=0, change=None, **options):
    """(bfloat16 patterns, the same as float arrays); change(name, values) may replace a tensor's values."""
    parsed = LayeredConfig.parse(cfg)
    patterns = parsed.random_tensors(np.random.default_rng(seed), **options)
    if change is not None:
        for name, array in patterns.items():
            new = change(name, from_bfloat16(array))
            if new is not None:
                patterns[name] = to_bfloat16(new)
    return patterns, {name: from_bfloat16(array).reshape(array.shape) for name, array in patterns.items()}


def make_model(runtime, cfg, patterns, dtype, **options):
    options.setdefault("max_context", 512)
    options.setdefault("slots", 3)
    return LayeredModel(runtime, LayeredConfig.parse(cfg), patterns, activations=dtype, **options)


def row_errors(actual, expected):
    """Root mean square of every row's difference over that of the expected array."""
    actual, expected = np.asarray(actual, np.float64), np.asarray(expected, np.float64)
    assert actual.shape == expected.shape, (actual.shape, expected.shape)
    assert np.all(np.isfinite(actual))
    return np.sqrt(np.mean((actual - expected) ** 2, axis=-1)) / np.sqrt(np.mean(expected ** 2))


def relative(actual, expected):
    return float(row_errors(actual, expected).max())


def assert_close(actual, expected, dtype, what=""):
    """float32: every row.  bfloat16: the median, and nine rows of ten - a router's close call or a row whose
    terms cancel in front of a norm shows the rounding of its operands many times over."""
    errors = row_errors(actual, expected)
    if dtype == "float32":
        assert errors.max() < 3e-5, (what, errors.max())
    else:
        assert np.median(errors) < 0.02 and np.quantile(errors, 0.9) < 0.06, (what, np.sort(errors)[-5:])


def run_portions(model, tokens, portions):
    """Logits of every token, fed in portions of the given sizes (repeated until the tokens are used up)."""
    sequence, rows, at, turn = model.open(), [], 0, 0
    while at < len(tokens):
        count = min(portions[turn % len(portions)], len(tokens) - at)
        rows.append(model.step(sequence, tokens[at:at + count], range(count)))
        at, turn = at + count, turn + 1
    model.close(sequence)
    return np.concatenate(rows)


def expected_logits(cfg, weights, tokens):
    return hybrid_model.forward(cfg, weights, tokens)[0]
