"""Decoders of the Koketar design on the GPU against the float64 restatement: every mechanism alone, prompts, decoding,
portions, window borders, the recurrence's memory, slots, and generation through the engine."""
import copy
import io
import json

import numpy as np
import pytest

from llmopt_amd import cli
from llmopt_amd.engine import Engine
from llmopt_amd.safetensors_file import write_safetensors
from oracle import parallel_model
from tests.layered_util import assert_close, make_model, make_weights, relative, run_portions
from tests.parallel_util import config, delta, dense, expected_logits, parallel, window

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]


@pytest.fixture(scope="module")
def runtime():
    from llmopt_amd.native import Runtime
    runtime = Runtime(device=0)
    yield runtime
    runtime.close()


def tokens_of(seed, count, vocab=90):
    return np.random.default_rng(2000 + seed).integers(0, vocab, count).tolist()


LEFT = {
    "window": window(),
    "one key head": window(heads=5, kv_heads=1, dim=32, vdim=32, size=7, rotated=32),
    "equal heads": window(heads=3, kv_heads=3, dim=16, vdim=8, size=200, rotated=8),
    "odd widths": window(heads=4, kv_heads=2, dim=13, vdim=27, size=33, rotated=12),
    "wide heads": window(heads=2, kv_heads=1, dim=136, vdim=200, size=64, scale=0.08, rotated=100),
    "many queries of a key head": window(heads=19, kv_heads=1, dim=16, vdim=24, size=30, rotated=16),
    "window of one": window(size=1),
    "window of two": window(size=2, rotated=2),
    "no scaling, low base": window(base=10.0, factor=1.0, rotated=24),
    "no window": {**window(), "mask": None},
    "no rotation": {**window(), "rot": None},
    "wide values, several splits": window(heads=4, kv_heads=2, dim=72, vdim=128, size=150, scale=0.1, rotated=40),
}
RIGHT = {
    "delta": delta(),
    "one head": delta(heads=1, kv_heads=1, dim=8, vdim=4),
    "equal heads": delta(heads=3, kv_heads=3, dim=32, vdim=16),
    "odd widths": delta(heads=4, kv_heads=2, dim=13, vdim=27),
    "one key head": delta(heads=5, kv_heads=1, dim=64, vdim=48),
    "wide keys": delta(heads=2, kv_heads=1, dim=100, vdim=64),
    "wide keys and odd values": delta(heads=1, kv_heads=1, dim=128, vdim=201),
    "wide": delta(heads=2, kv_heads=2, dim=128, vdim=128),
    "widest": delta(heads=1, kv_heads=1, dim=256, vdim=256),
    "one tap": delta(conv=1),
    "two taps": delta(conv=2),
    "seven taps": delta(conv=7),
}


def check_streams(runtime, cfg, dtype, count=75, seed=0, change=None, **options):
    patterns, weights = make_weights(cfg, seed, change, **options)
    model = make_model(runtime, cfg, patterns, dtype)
    tokens = tokens_of(seed, count, cfg["vocab"])
    expected, streams = parallel_model.forward(cfg, weights, tokens)
    sequence, got = model.open(), []
    logits = model.step(sequence, tokens, range(count), streams=got)
    model.close(sequence)
    for index, stream in enumerate(got):
        assert_close(stream, streams[index], dtype, f"prompt, layer {index}")
    assert_close(logits, expected, dtype)
    sequence = model.open()
    decoded = np.concatenate([model.step(sequence, [t], [0]) for t in tokens])
    model.close(sequence)
    assert_close(decoded, expected, dtype, "token by token")


def only(side):
    """One of the two mixers alone: the other one's scale is zero."""
    return {"left_scale": 1.1, "right_scale": 0.0} if side == "left" else {"left_scale": 0.0, "right_scale": 1.1}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(LEFT))
def test_window_attention_alone(runtime, name, dtype):
    print(name, dtype, flush=True)
    check_streams(runtime, config(parallel(left=LEFT[name], **only("left"))), dtype, count=170 if "splits" in name else 75)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(RIGHT))
def test_gated_delta_alone(runtime, name, dtype):
    print(name, dtype, flush=True)
    check_streams(runtime, config(parallel(right=RIGHT[name], **only("right"))), dtype, rank=9 if "odd" in name else 16)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("limit", [0.05, 1.0, 100.0])
@pytest.mark.parametrize("ff", [104, 57])
def test_feed_forward_alone(runtime, ff, limit, dtype):
    """The limits reached by nearly all, some, and no values; the mixer's norm weights make it next to nothing."""
    print(ff, limit, dtype, flush=True)
    small = lambda name, values: values * 0.0 - 0.98 if name == "l0.norm1" else None
    check_streams(runtime, config(parallel(mlp=dense(ff, limit))), dtype, count=40, change=small)


CONFIGS = {
    "two layers": config(parallel(mlp=dense()), parallel(mlp=dense(200, 3.0))),
    "some without a feed-forward": config(parallel(), parallel(window(size=9), delta(conv=3), mlp=dense()), parallel()),
    "all different": config(parallel(window(heads=2, kv_heads=1, size=50), delta(heads=6, kv_heads=3, dim=33, vdim=12), 0.3,
                                     1.2, dense(40, 0.4)),
                            parallel(window(heads=8, kv_heads=4, dim=16, vdim=16, size=5, rotated=4),
                                     delta(heads=2, kv_heads=1, dim=40, vdim=80, conv=2), 1.5, 0.2, dense(90, 2.0)),
                            vocab=131, width=100, mult=1.3, softcap=5.0, eps=1e-3),
    "odd width": config(parallel(mlp=dense(50)), parallel(mlp=dense(33)), width=61, vocab=77),
    "no cap on the logits": config(parallel(mlp=dense()), softcap=None),
    "aligned": config(parallel(window(heads=4, kv_heads=2, dim=64, vdim=64, rotated=64), delta(2, 2, 64, 64), mlp=dense(256)),
                      width=128, vocab=256),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_layers_together(runtime, name, dtype):
    print(name, dtype, flush=True)
    cfg = CONFIGS[name]
    restated = copy.deepcopy(cfg)
    if cfg["logit_softcap"] is None:
        restated["logit_softcap"] = 1e9
    patterns, weights = make_weights(cfg, 3, rank=64 if name == "aligned" else 12)
    model = make_model(runtime, cfg, patterns, dtype)
    tokens = tokens_of(3, 90, cfg["vocab"])
    expected, streams = parallel_model.forward(restated, weights, tokens)
    sequence, got = model.open(), []
    assert_close(model.step(sequence, tokens, range(90), streams=got), expected, dtype)
    model.close(sequence)
    for index, stream in enumerate(got):
        assert_close(stream, streams[index], dtype, index)
    assert_close(run_portions(model, tokens, [1]), expected, dtype)


@pytest.fixture(scope="module")
def mixed():
    cfg = config(parallel(window(size=24), mlp=dense()), parallel(window(heads=3, kv_heads=3, size=70), delta(conv=3)),
                 parallel(window(size=11), delta(heads=2, kv_heads=2, dim=24, vdim=36), mlp=dense(88, 2.0)))
    patterns, weights = make_weights(cfg, 5)
    tokens = tokens_of(5, 210)
    return cfg, patterns, weights, tokens, expected_logits(cfg, weights, tokens)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("portions", [[210], [2], [3, 64], [1], [24], [17, 1, 2], [100, 1, 1, 9], [65, 63, 2]])
def test_portions(runtime, mixed, portions, dtype):
    cfg, patterns, _, tokens, expected = mixed
    print(portions, dtype, flush=True)
    model = make_model(runtime, cfg, patterns, dtype)
    assert_close(run_portions(model, tokens, portions), expected, dtype)


def test_slots_are_reused_and_do_not_leak(runtime, mixed):
    """Sequences of unequal lengths interleaved on three slots, closed and opened again: each as if alone."""
    cfg, patterns, weights, _, _ = mixed
    model = make_model(runtime, cfg, patterns, "float32")
    prompts = [tokens_of(20 + i, n) for i, n in enumerate((40, 3, 77, 1, 26, 110, 2))]
    expected = [expected_logits(cfg, weights, p) for p in prompts]
    waiting, live, rng = list(range(len(prompts))), {}, np.random.default_rng(7)
    while waiting or live:
        while waiting and model.state.free_slots:
            live[waiting.pop(0)] = [model.open(), 0]
        index = int(rng.choice(sorted(live)))
        sequence, at = live[index]
        count = min(int(rng.integers(1, 30)), len(prompts[index]) - at)
        logits = model.step(sequence, prompts[index][at:at + count], range(count))
        assert_close(logits, expected[index][at:at + count], "float32", (index, at, count))
        live[index][1] += count
        if live[index][1] == len(prompts[index]):
            model.close(sequence)
            del live[index]


def needle_model(size):
    """Two attention heads alone; token 0 is the query, token 1 a key that outscores everything wherever it stands (its
    large components do not rotate)."""
    cfg = config(parallel(window(heads=2, kv_heads=1, dim=16, vdim=24, size=size, scale=2.0, rotated=4), delta(), 1.0, 0.0),
                 width=64, vocab=50, softcap=60.0)

    def change(name, values):
        if name == "embed":
            values[:, :16] = 0.0
            values[0, 0] = 6.0
            values[1, 1] = 6.0
        if name == "l0.mix.left.q":
            values *= 0.1
            values[[8, 24], 0] = 8.0
        if name == "l0.mix.left.k":
            values *= 0.1
            values[8, 1] = 8.0
        if name.endswith(("q.norm", "k.norm")):
            values[:] = 1.0
        return values
    return cfg, change


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size", [16, 33, 64, 129, 300])
def test_window_edges(runtime, size, dtype):
    """One key stands out: the first that a query sees, the last that it no longer sees, or far back among hundreds."""
    cfg, change = needle_model(size)
    patterns, weights = make_weights(cfg, 2, change)
    model = make_model(runtime, cfg, patterns, dtype, max_context=1024)
    filler = np.random.default_rng(9).integers(2, 50, 2 * size + 40)
    key = 19
    tokens = filler.copy()
    tokens[key] = 1
    queries = [key + 1, key + size - 2, key + size - 1, key + size, key + size + 1, key + size + 17]
    tokens[queries] = 0
    tokens = tokens.tolist()
    expected = expected_logits(cfg, weights, tokens)
    for portions in ([len(tokens)], [key + size - 1, 1, 1], [key + 1, size - 2, 1, 3], [64], [1]):
        print(size, portions, dtype, flush=True)
        assert_close(run_portions(model, tokens, portions), expected, dtype, (size, portions))
    # a window that is one token off shows at the queries on its edge
    for wrong, place in ((size - 1, key + size - 1), (size + 1, key + size)):
        shifted = copy.deepcopy(cfg)
        shifted["layers"][0]["mixer"]["left"]["mask"]["size"] = wrong
        off = expected_logits(shifted, weights, tokens)
        assert relative(off[[place]], expected[[place]]) > 0.3, (wrong, place)


@pytest.mark.parametrize("dtype", DTYPES)
def test_positions_of_a_rotation(runtime, dtype):
    """Full rotation with large scores: the logits depend on distances far apart, across portions and in decoding."""
    cfg = config(parallel(window(heads=2, kv_heads=2, dim=16, vdim=24, size=250, scale=1.5, rotated=16, base=40.0, factor=2.0),
                          delta(), 1.0, 0.0))
    patterns, weights = make_weights(cfg, 12)
    tokens = tokens_of(12, 260)
    expected = expected_logits(cfg, weights, tokens)
    model = make_model(runtime, cfg, patterns, dtype)
    for portions in ([260], [97, 2, 1], [1]):
        assert_close(run_portions(model, tokens, portions), expected, dtype, portions)
    unscaled = copy.deepcopy(cfg)
    unscaled["layers"][0]["mixer"]["left"]["rot"]["scaling"]["factor"] = 1.0
    assert relative(expected_logits(unscaled, weights, tokens), expected) > 0.1


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_memory_of_the_recurrence(runtime, dtype):
    """Decays so slow that a state remembers hundreds of tokens, so fast that nothing survives one, and both in one head,
    over several chunks of the scan and in long decoding."""
    cfg = config(parallel(right=delta(heads=6, kv_heads=3, dim=48, vdim=32), **only("right")))

    def change(name, values):
        if name.endswith("A_log"):
            return np.array([-7.0, -5.0, -2.0, 1.0, 3.0, 0.0])
        if name.endswith("dt_bias"):
            return np.where(np.arange(values.size) % 48 < 24, 3.0, -6.0)
        return None
    patterns, weights = make_weights(cfg, 6, change)
    model = make_model(runtime, cfg, patterns, dtype)
    tokens = tokens_of(6, 300)
    expected = expected_logits(cfg, weights, tokens)
    for portions in ([300], [70, 1, 1], [2], [1]):
        print(portions, dtype, flush=True)
        assert_close(run_portions(model, tokens, portions), expected, dtype, portions)
    # the memory is there: other first tokens show hundreds of tokens later
    other = expected_logits(cfg, weights, tokens_of(66, 30) + tokens[30:])
    assert relative(other[[280]], expected[[280]]) > 1e-3


@pytest.mark.parametrize("dtype", DTYPES)
def test_repeated_keys_are_overwritten(runtime, dtype):
    """Full write strengths on the same two tokens over and over: the triangular solves' worst case."""
    cfg = config(parallel(right=delta(heads=2, kv_heads=1, dim=16, vdim=24, conv=1), **only("right")))

    def change(name, values):
        if name.endswith("A_log"):
            return np.full(values.shape, -6.0)
        if name == "l0.mix.right.b":
            return values * 6.0
        return None
    patterns, weights = make_weights(cfg, 13, change)
    model = make_model(runtime, cfg, patterns, dtype)
    tokens = ([3, 7] * 70 + [11, 3])[:141]
    expected = expected_logits(cfg, weights, tokens)
    for portions in ([141], [64, 3], [1]):
        assert_close(run_portions(model, tokens, portions), expected, dtype, portions)


@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens(runtime, mixed, dtype):
    """Before the convolution's and the window's full length; a second sequence on a used slot starts afresh."""
    cfg, patterns, _, tokens, expected = mixed
    model = make_model(runtime, cfg, patterns, dtype, slots=1)
    run_portions(model, tokens_of(71, 40), [40])
    for count in (1, 2, 3, 4, 5):
        assert_close(run_portions(model, tokens[:count], [count]), expected[:count], dtype)
        assert_close(run_portions(model, tokens[:count], [1]), expected[:count], dtype)


def greedy(cfg, weights, prompt, count):
    tokens = list(prompt)
    for _ in range(count):
        tokens.append(int(np.argmax(expected_logits(cfg, weights, tokens)[-1])))
    return tokens[len(prompt):]


def test_greedy_generation_through_the_engine(runtime, mixed):
    """More requests than slots, prompts longer than a portion, against argmax of the restatement."""
    cfg, patterns, weights, _, _ = mixed
    model = make_model(runtime, cfg, patterns, "float32", slots=2)
    prompts = [tokens_of(40 + i, n) for i, n in enumerate((30, 1, 12, 19))]
    got = Engine(model, portion=8).generate(prompts, max_new_tokens=9)
    assert got == [greedy(cfg, weights, p, 9) for p in prompts]
    assert model.state.free_slots == 2


def test_long_generation_is_what_a_prompt_of_it_gives(runtime, mixed):
    """200 tokens decoded through the captured graph; the whole text as one prompt has the same logits."""
    cfg, patterns, _, _, _ = mixed
    model = make_model(runtime, cfg, patterns, "float32")
    prompt = tokens_of(45, 9)
    text = prompt + Engine(model).generate([prompt], 200)[0]
    sequence = model.open()
    logits = model.step(sequence, text, range(len(text)))
    model.close(sequence)
    assert logits[len(prompt) - 1:-1].argmax(1).tolist() == text[len(prompt):]
    assert model.decode_plan().plan.single_submission


def test_a_plan_replays_like_eager_steps(runtime, mixed):
    """The captured graph, many times, with portions of another sequence in between."""
    cfg, patterns, _, tokens, expected = mixed
    model = make_model(runtime, cfg, patterns, "float32")
    sequences, at = (model.open(), model.open()), [0, 0]
    for turn in range(60):
        which = turn % 2
        count = 1 if turn % 5 else 3
        part = tokens[at[which]:at[which] + count]
        got = model.step(sequences[which], part, range(count))
        assert_close(got, expected[at[which]:at[which] + count], "float32", turn)
        at[which] += count


def test_one_token_step_with_its_streams(runtime, mixed):
    """A single token outside the plan, asked for twice."""
    cfg, patterns, weights, tokens, expected = mixed
    model = make_model(runtime, cfg, patterns, "float32")
    streams, sequence = [], model.open()
    logits = model.step(sequence, tokens[:1], [0, 0], streams=streams)
    assert_close(logits, expected[[0, 0]], "float32")
    for got, want in zip(streams, parallel_model.forward(cfg, weights, tokens[:1])[1]):
        assert_close(got, want, "float32")


def test_command_line(runtime, mixed, tmp_path, capsys, monkeypatch):
    """A model folder through `generate` and `replay`."""
    cfg, patterns, weights, tokens, expected = mixed
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    write_safetensors(str(tmp_path / "model.safetensors"), patterns)
    prompt = tokens_of(60, 11)
    assert cli.main(["generate", "--model", str(tmp_path), "--dtype", "float32", "--max-new-tokens", "5",
                     "--max-context", "64", "--prompt", ",".join(map(str, prompt))]) == 0
    assert [int(t) for t in capsys.readouterr().out.split()] == greedy(cfg, weights, prompt, 5)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": tokens[:20], "want": [3, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": tokens[20:21], "want": [0]}], "end": ["a"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n"))
    out = tmp_path / "out"
    assert cli.main(["replay", "--model", str(tmp_path), "--dtype", "float32", "--out", str(out),
                     "--max-tokens", "64"]) == 0
    assert capsys.readouterr().out.split("\n")[:2] == ["done 0", "done 1"]
    read = lambda n, rows: np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(rows, -1)
    assert_close(read(0, 2), expected[[3, 19]], "float32")
    assert_close(read(1, 1), expected[[20]], "float32")


@pytest.mark.parametrize("dtype", DTYPES)
def test_sizes_of_a_real_layer(runtime, dtype):
    """The large tiles, direct copies and several rounds of splits, checked on a sample of rows."""
    cfg = config(parallel(window(heads=8, kv_heads=2, dim=128, vdim=128, size=200, scale=0.09, rotated=64),
                          delta(heads=4, kv_heads=4, dim=128, vdim=128), mlp=dense(2048, 4.0)), vocab=3000, width=1024)
    patterns, weights = make_weights(cfg, 8, rank=128)
    model = make_model(runtime, cfg, patterns, dtype, max_context=1024)
    tokens = tokens_of(8, 330, 3000)
    expected, streams = parallel_model.forward(cfg, weights, tokens)
    got, sequence, wanted = [], model.open(), [0, 1, 199, 200, 329]
    logits = model.step(sequence, tokens, wanted, streams=got)
    assert_close(got[0], streams[0], dtype)
    assert_close(logits, expected[wanted], dtype)
    sequence = model.open()
    model.step(sequence, tokens[:320])
    decoded = np.concatenate([model.step(sequence, [t], [0]) for t in tokens[320:]])
    assert_close(decoded, expected[320:], dtype)


def test_entries_refuse_what_does_not_fit(runtime, mixed):
    """Sizes are checked on the host, before anything is launched."""
    from llmopt_amd.native import DispatchList, LlmoptError
    cfg, patterns, _, _, _ = mixed
    model = make_model(runtime, cfg, patterns, "float32")
    plan = model.decode_plan()
    for name, buffers, parameters, grid, group in plan.dispatches:
        if not name.startswith(("llmopt_joint", "llmopt_rotary", "llmopt_gated_delta", "llmopt_pending", "llmopt_linear_store")):
            continue
        grown = np.frombuffer(parameters, np.uint32).copy()
        grown[1] *= 64  # the width, or the heads, or the rows of the product
        batch = runtime.begin_batch()
        with pytest.raises(LlmoptError):
            batch.dispatch_all(DispatchList([(name, buffers, grown.tobytes(), grid, group)]))
            batch.commit()
