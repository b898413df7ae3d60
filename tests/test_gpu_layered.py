"""Layered decoders on the GPU against the float64 restatement: every mechanism alone, prompts, decoding,
portions, chunk borders, slots, and generation through the engine."""
import copy

import numpy as np
import pytest

from llmopt_amd.engine import Engine
from oracle import hybrid_model
from tests.layered_util import (assert_close, attention, config, dense, expected_logits, make_model, make_weights, mamba2,
                                moe, relative, run_portions)

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]


@pytest.fixture(scope="module")
def runtime():
    from llmopt_amd.native import Runtime
    runtime = Runtime(device=0)
    yield runtime
    runtime.close()


def tokens_of(seed, count, vocab=90):
    return np.random.default_rng(1000 + seed).integers(0, vocab, count).tolist()


MECHANISMS = {
    "attention": attention(),
    "attention one kv head": attention(heads=5, kv_heads=1, dim=32, vdim=32, chunk=7),
    "attention equal heads": attention(heads=3, kv_heads=3, dim=16, vdim=8, chunk=100),
    "attention odd widths": attention(heads=4, kv_heads=2, dim=13, vdim=27, chunk=33),
    "attention wide heads": attention(heads=2, kv_heads=1, dim=136, vdim=200, chunk=64, scale=0.08),
    "attention wide values": attention(heads=4, kv_heads=1, dim=72, vdim=128, chunk=50, scale=0.1),
    "attention large cap": attention(softcap=90.0, scale=1.0),
    "attention no cap": attention(softcap=None),
    "attention no chunks": attention(chunk=1 << 20),
    "mamba2": mamba2(),
    "mamba2 one group": mamba2(heads=5, vdim=16, state=32, groups=1, norm_groups=1),
    "mamba2 group per head": mamba2(heads=4, vdim=33, state=17, groups=4, norm_groups=2, conv=3),
    "mamba2 state of 128": mamba2(heads=2, vdim=64, state=128, groups=1, norm_groups=4, conv=2),
    "mamba2 state of 200": mamba2(heads=2, vdim=8, state=200, groups=2, norm_groups=1, conv=6),
    "mamba2 one tap": mamba2(conv=1),
}
FEED_FORWARDS = {
    "dense": dense(),
    "dense odd": dense(ff=57),
    "experts": moe(),
    "experts, no shared": moe(experts=9, top=3, ff=33, shared=0),
    "one of many": moe(experts=70, top=1, ff=16, shared=24),
    "all of them": moe(experts=4, top=4, ff=64, shared=8),
}


def check_streams(runtime, cfg, dtype, count=75, seed=0, change=None):
    patterns, weights = make_weights(cfg, seed, change)
    model = make_model(runtime, cfg, patterns, dtype)
    tokens = tokens_of(seed, count, cfg["vocab"])
    expected, streams = hybrid_model.forward(cfg, weights, tokens)
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


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MECHANISMS))
def test_mixer_alone(runtime, name, dtype):
    print(name, dtype, flush=True)
    check_streams(runtime, config(MECHANISMS[name]), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(FEED_FORWARDS))
def test_feed_forward_alone(runtime, name, dtype):
    print(name, dtype, flush=True)
    # a mixer of almost nothing in front, so that the feed-forward is what shows
    small = lambda tensor, values: values * 0.02 if tensor.endswith("mix.o") else None
    check_streams(runtime, config(attention(heads=1, kv_heads=1, dim=8, vdim=8, mlp=FEED_FORWARDS[name])), dtype,
                  count=40, change=small)


ORDERS = {
    "alternating": config(mamba2(mlp=dense()), attention(mlp=moe()), mamba2(mlp=dense(96)), attention(mlp=moe())),
    "attention first": config(attention(mlp=moe(top=3)), attention(v_mix=False, vdim=24, mlp=None),
                              mamba2(mlp=moe(experts=3, top=1)), attention(chunk=11, mlp=dense()), mamba2(),
                              vocab=131, width=100),
    "odd width": config(mamba2(mlp=dense(50)), attention(mlp=moe(ff=30, shared=21)), width=61, vocab=77),
    "recurrent only": config(mamba2(mlp=dense()), mamba2(groups=3, norm_groups=6)),
    "attention only": config(attention(mlp=dense()), attention(kv_heads=3, chunk=9, mlp=dense()), attention()),
}


def all_chosen(cfg):
    """The same with every expert chosen: no close call for bfloat16 to decide the other way."""
    cfg = copy.deepcopy(cfg)
    for layer in cfg["layers"]:
        if layer["mlp"] and layer["mlp"]["kind"] == "moe":
            layer["mlp"]["router"]["top"] = layer["mlp"]["router"]["experts"]
    return cfg


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(ORDERS))
def test_layer_orders(runtime, name, dtype):
    print(name, dtype, flush=True)
    cfg = ORDERS[name] if dtype == "float32" else all_chosen(ORDERS[name])
    check_streams(runtime, cfg, dtype, count=90, seed=3)


@pytest.mark.parametrize("dtype", DTYPES)
def test_value_mix_of_several_layers(runtime, dtype):
    """Three mixing layers with strong, different lambdas and one that does not mix in between."""
    lambdas = {"l0.mix.vmix": 0.9, "l2.mix.vmix": 0.75, "l3.mix.vmix": 0.25}
    cfg = config(attention(), attention(v_mix=False), attention(chunk=13), attention(heads=3))
    check_streams(runtime, cfg, dtype, change=lambda name, values: lambdas.get(name))


def mixed_model(top):
    cfg = config(mamba2(mlp=dense()), attention(chunk=24, mlp=moe(top=top)), mamba2(vdim=10, mlp=moe(top=top, shared=0)),
                 attention(chunk=17, heads=3, mlp=dense()))
    patterns, weights = make_weights(cfg, 5)
    tokens = tokens_of(5, 210)
    return cfg, patterns, weights, tokens, expected_logits(cfg, weights, tokens)


@pytest.fixture(scope="module")
def mixed():
    return mixed_model(top=2)


@pytest.fixture(scope="module")
def mixed_all():
    """Every expert is chosen (see all_chosen)."""
    return mixed_model(top=6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("portions", [[210], [2], [3, 64], [1], [24], [17, 1, 2], [100, 1, 1, 9], [65, 63, 2]])
def test_portions(runtime, mixed, mixed_all, portions, dtype):
    cfg, patterns, _, tokens, expected = mixed if dtype == "float32" else mixed_all
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


def needle_model(chunk, sink=-4.0):
    """Two attention heads; token 0 is the query, token 1 a key that outscores everything by the full cap."""
    cfg = config(attention(heads=2, kv_heads=1, dim=16, vdim=24, chunk=chunk, scale=1.0, softcap=12.0, v_mix=False),
                 width=64, vocab=50)

    def change(name, values):
        if name == "embed":
            values[:, :16] = 0.0
            values[0, 0] = 6.0
            values[1, 1] = 6.0
        if name == "l0.norm1":
            values[:] = 1.0
        if name == "l0.mix.q":
            values[:] = 0.0
            values[[0, 16], 0] = 8.0
        if name == "l0.mix.k":
            values[:] = 0.0
            values[0, 1] = 8.0
        if name == "l0.mix.sink":
            values[:] = sink
        return values
    return cfg, change


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunk", [16, 33, 64, 130])
def test_chunk_edges(runtime, chunk, dtype):
    """One key stands out.  It is the last of a chunk, the first of the next one, or far back in the same chunk;
    seen or not changes the output by more than its size."""
    cfg, change = needle_model(chunk)
    patterns, weights = make_weights(cfg, 2, change)
    model = make_model(runtime, cfg, patterns, dtype)
    filler = np.random.default_rng(9).integers(2, 50, 3 * chunk)
    shifted = copy.deepcopy(cfg)
    for place in (0, chunk - 1, chunk, chunk + 1, 2 * chunk - 1):
        tokens = filler.copy()
        tokens[place] = 1
        tokens[[chunk - 2, chunk, 2 * chunk - 1, 2 * chunk, 3 * chunk - 1]] = 0
        tokens[place] = 1
        tokens = tokens.tolist()
        expected = expected_logits(cfg, weights, tokens)
        print(chunk, place, dtype, flush=True)
        for portions in ([3 * chunk], [chunk - 1, 2], [chunk + 1, 1, 3], [1]):
            got = run_portions(model, tokens, portions)
            assert_close(got, expected, dtype, (place, portions))
    # the comparison would notice a border that is one token off
    tokens = filler.copy()
    tokens[chunk - 1], tokens[chunk] = 1, 0
    for wrong in (chunk - 1, chunk + 1):
        shifted["layers"][0]["mixer"]["mask"]["size"] = wrong
        off = expected_logits(shifted, weights, tokens.tolist())
        assert relative(off, expected_logits(cfg, weights, tokens.tolist())) > 0.3


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_key_and_sink_over_many_splits(runtime, dtype):
    """Decoding deep inside a long chunk: one far key among hundreds, with and without a heavy sink."""
    for sink in (-4.0, 9.0):
        cfg, change = needle_model(400, sink)
        patterns, weights = make_weights(cfg, 4, change)
        model = make_model(runtime, cfg, patterns, dtype)
        tokens = np.random.default_rng(11).integers(2, 50, 390)
        tokens[5] = 1
        tokens[[6, 127, 128, 255, 256, 300, 383, 389]] = 0
        expected = expected_logits(cfg, weights, tokens.tolist())
        for portions in ([390], [383, 1], [120, 1, 1, 1, 1, 1, 1, 1, 1, 1, 1]):
            assert_close(run_portions(model, tokens.tolist(), portions), expected, dtype, (sink, portions))
        without = {**weights, "l0.mix.sink": np.full(2, -30.0)}
        if sink > 0:
            assert relative(expected_logits(cfg, without, tokens.tolist()), expected) > 0.3


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_memory_of_the_recurrence(runtime, dtype):
    """Slow decays (a state that remembers hundreds of tokens) and fast ones (differences of large running
    sums), over several chunks of the scan and in long decoding."""
    cfg = config(mamba2(heads=8, vdim=16, state=48, groups=2, norm_groups=2))

    def change(name, values):
        if name.endswith("A_log"):
            return np.array([-7.0, -6.0, -4.0, -2.0, 0.0, 1.0, 2.0, 3.0])
        if name.endswith("dt_bias"):
            return np.array([1.0, 0.0, 1.0, 0.0, 2.0, 3.0, 4.0, 4.0])
        if name.endswith("mix.D"):
            return values * 0.1
        return None
    patterns, weights = make_weights(cfg, 6, change)
    model = make_model(runtime, cfg, patterns, dtype)
    tokens = tokens_of(6, 300)
    expected = expected_logits(cfg, weights, tokens)
    for portions in ([300], [70, 1, 1], [2], [1]):
        print(portions, dtype, flush=True)
        assert_close(run_portions(model, tokens, portions), expected, dtype, portions)


def test_first_tokens(runtime, mixed):
    cfg, patterns, _, tokens, expected = mixed
    model = make_model(runtime, cfg, patterns, "float32")
    for count in (1, 2, 3, 4, 5):
        assert_close(run_portions(model, tokens[:count], [count]), expected[:count], "float32")
        assert_close(run_portions(model, tokens[:count], [1]), expected[:count], "float32")


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


def test_generation_with_other_settings(runtime, mixed):
    from llmopt_amd.sampling import Params
    cfg, patterns, weights, _, _ = mixed
    model = make_model(runtime, cfg, patterns, "float32")
    prompt = tokens_of(50, 14)
    engine = Engine(model)
    want = greedy(cfg, weights, prompt, 6)
    assert engine.generate([prompt], 6, stop_tokens=[want[2]])[0] == want[:want.index(want[2]) + 1]
    seeded = Params.create(temperature=1.0, top_k=20, seed=77)
    first, second = engine.generate([prompt, prompt], 12, seeded)
    assert first == second and first != engine.generate([prompt], 12, Params.create(1.0, 20, seed=78))[0]


def test_a_plan_replays_like_eager_steps(runtime, mixed):
    """The captured graph, many times, with other work on the stream in between."""
    cfg, patterns, _, tokens, expected = mixed
    model = make_model(runtime, cfg, patterns, "float32")
    one, two = model.open(), model.open()
    at = {0: 0, 1: 0}
    for turn in range(60):
        which = turn % 2
        sequence = (one, two)[which]
        count = 1 if turn % 5 else 3
        part = tokens[at[which]:at[which] + count]
        got = model.step(sequence, part, range(count))
        assert_close(got, expected[at[which]:at[which] + count], "float32", turn)
        at[which] += count
    assert model.decode_plan().plan.single_submission


def test_limits_are_errors(runtime, mixed):
    from llmopt_amd.native import LlmoptError
    from llmopt_amd.sequence_state import StateError
    cfg, patterns, _, tokens, _ = mixed
    model = make_model(runtime, cfg, patterns, "float32", slots=1, max_context=32)
    sequence = model.open()
    with pytest.raises(StateError):
        model.open()
    with pytest.raises(StateError):
        model.step(sequence, tokens[:33])
    with pytest.raises(ValueError):
        model.step(sequence, [90])
    with pytest.raises(ValueError):
        model.step(sequence, [1, 2], [2])
    model.step(sequence, tokens[:32])
    with pytest.raises(StateError):
        model.decode(sequence, 0)
    with pytest.raises(LlmoptError):
        model.decode_plan().plan.execute(0, 40, 0)   # beyond the pool's context
    with pytest.raises(LlmoptError):
        model.decode_plan().plan.execute(0, 3, 1)    # no such slot
    model.close(sequence)
    with pytest.raises(StateError):
        model.step(sequence, tokens[:2])


def test_command_line(runtime, mixed, tmp_path, capsys, monkeypatch):
    """A model folder through `generate` and `replay`."""
    import io
    import json

    from llmopt_amd import cli
    from llmopt_amd.safetensors_file import write_safetensors
    cfg, patterns, weights, tokens, expected = mixed
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    write_safetensors(str(tmp_path / "model.safetensors"), patterns)
    prompt = tokens_of(60, 11)
    assert cli.main(["generate", "--model", str(tmp_path), "--dtype", "float32", "--max-new-tokens", "5",
                     "--max-context", "64", "--prompt", ",".join(map(str, prompt))]) == 0
    assert [int(t) for t in capsys.readouterr().out.split()] == greedy(cfg, weights, prompt, 5)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": tokens[:20], "want": [3, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": tokens[20:21], "want": [0]}], "end": ["a"]},
             {"step": 2, "entries": [{"id": "b", "tokens": tokens[:2], "want": []}], "end": ["b"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n"))
    out = tmp_path / "out"
    assert cli.main(["replay", "--model", str(tmp_path), "--dtype", "float32", "--out", str(out),
                     "--max-tokens", "64"]) == 0
    assert capsys.readouterr().out.split("\n")[:3] == ["done 0", "done 1", "done 2"]
    read = lambda n, rows: np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(rows, -1)
    assert_close(read(0, 2), expected[[3, 19]], "float32")
    assert_close(read(1, 1), expected[[20]], "float32")
    assert not (out / "2.f32").exists()


@pytest.mark.parametrize("dtype", DTYPES)
def test_sizes_of_a_real_layer(runtime, dtype):
    """The large tiles: a prompt long enough for the 128-row products, checked on a sample of rows."""
    cfg = config(mamba2(heads=16, vdim=64, state=128, groups=1, norm_groups=1, mlp=dense(2048)),
                 attention(heads=8, kv_heads=2, dim=128, vdim=128, chunk=256, scale=0.09, mlp=moe(8, 2, 512, 512)),
                 vocab=3000, width=1024)
    patterns, weights = make_weights(cfg, 8)
    model = make_model(runtime, cfg, patterns, dtype, max_context=1024)
    tokens = tokens_of(8, 330, 3000)
    got = []
    sequence = model.open()
    logits = model.step(sequence, tokens, [0, 1, 255, 256, 329], streams=got)
    # the recurrence alone is slow to restate at this size: the first layer over all tokens is enough for both
    expected, streams = hybrid_model.forward(cfg, weights, tokens)
    for index in range(2):
        assert_close(got[index], streams[index], dtype, index)
    assert_close(logits, expected[[0, 1, 255, 256, 329]], dtype)
