"""Host side of the layered decoders without a GPU: configuration, weight files, state slots, the
scheduler over a model of plain Python, the float32 sampler, and the restatement's own consistency."""
import io
import json

import numpy as np
import pytest

from llmopt_amd import model_registry, sampling, trace_replay
from llmopt_amd.engine import Engine
from llmopt_amd.layered_model import (DESIGNS, AttentionMixer, DeltaMixer, DenseFfn, JointColumns, LayeredConfig, LayeredModel,
                                      Mamba2Mixer, RoutedFfn, Rotation, WindowMixer, _Tensors)
from llmopt_amd.safetensors_file import (SafetensorsError, SafetensorsFile, from_bfloat16, to_bfloat16,
                                         write_safetensors)
from llmopt_amd.sequence_state import RingShape, Sequence, StateError, StatePool
from oracle import hybrid_model, parallel_model
from tests import parallel_util as pu
from tests.layered_util import attention, config, dense, make_weights, mamba2, moe


def test_config_reads_every_size():
    parsed = LayeredConfig.parse(config(mamba2(mlp=dense(7)), attention(mlp=moe(5, 2, 8, 9)), attention(softcap=None)))
    assert parsed.layers[0].mixer == Mamba2Mixer(6, 20, 24, 2, 4, 3) and parsed.layers[0].ffn == DenseFfn(7)
    assert parsed.layers[1].mixer == AttentionMixer(6, 3, 24, 40, 0.3, 8.0, 20, True)
    assert parsed.layers[1].ffn == RoutedFfn(5, 2, 8, 9)
    assert parsed.layers[2].mixer.softcap == 0.0 and parsed.layers[2].ffn is None
    shapes = parsed.tensor_shapes()
    assert shapes["l0.mix.in"] == (2 * 120 + 2 * 48 + 6, 72) and shapes["l0.mix.conv"] == (216, 4)
    assert shapes["l1.mlp.e4.down"] == (72, 8) and shapes["l1.mlp.shared.sg"] == (1, 72)
    assert "l2.norm2" not in shapes and shapes["l1.mix.vmix"] == ()


@pytest.mark.parametrize("bad", [
    config({"type": "other", "mixer": {}, "mlp": None}),
    config(attention(mlp={"kind": "other"})),
    config(attention(heads=5, kv_heads=2)),
    config(mamba2(heads=5, groups=2)),
    config(mamba2(norm_groups=7)),
    config(attention(), attention(vdim=8)),
])
def test_config_refuses(bad):
    with pytest.raises(ValueError):
        LayeredConfig.parse(bad)


def test_registry(tmp_path):
    assert model_registry.model_class({"architecture": "Barovik"}) is LayeredModel
    assert "Barovik" in model_registry.architectures()
    with pytest.raises(model_registry.UnknownArchitecture):
        model_registry.model_class({"architecture": "nothing"})


def test_safetensors_round_trip_and_checks(tmp_path):
    path = str(tmp_path / "w.safetensors")
    values = np.array([1.0, -2.5, 3.1415926, 1e-30], dtype=np.float32)
    write_safetensors(path, {"a": to_bfloat16(values), "s": to_bfloat16(0.5), "t": np.arange(6, dtype=np.int32).reshape(2, 3)})
    file = SafetensorsFile(path)
    assert np.allclose(from_bfloat16(file.bfloat16("a", (4,))), values, rtol=2 ** -8)
    assert file.bfloat16("s", ()).shape == () and file.numpy("t").tolist() == [[0, 1, 2], [3, 4, 5]]
    for call in (lambda: file.bfloat16("a", (2, 2)), lambda: file.bfloat16("t", (2, 3)), lambda: file.numpy("b")):
        with pytest.raises(SafetensorsError):
            call()
    raw = open(path, "rb").read()
    open(path, "wb").write(raw[:-3])
    with pytest.raises(SafetensorsError):
        SafetensorsFile(path)


def test_bfloat16_rounds_to_nearest_even():
    assert to_bfloat16(np.float32(1.0 + 2 ** -8)) == to_bfloat16(np.float32(1.0))
    assert to_bfloat16(np.float32(1.0 + 3 * 2 ** -8)) == to_bfloat16(np.float32(1.0 + 2 ** -6))


class FakeRuntime:
    def __init__(self):
        self.sizes = []

    def create_buffer(self, size):
        self.sizes.append(size)
        return size


def test_state_pool():
    assert RingShape.of(2, 8, 4, 16, 100) == RingShape(2, 8, 4, 16, 16)
    assert RingShape.of(2, 8, 4, 0, 100) == RingShape.of(2, 8, 4, 100, 100) == RingShape(2, 8, 4, 0, 100)
    runtime = FakeRuntime()
    pool = StatePool(runtime, [(RingShape.of(2, 8, 4, 16, 100),)], slots=2, max_context=100, element_bytes=2)
    assert runtime.sizes == [2 * 2 * 16 * 2 * 8, 2 * 2 * 16 * 2 * 4]
    a, b = pool.open(), pool.open()
    assert a.slot != b.slot and pool.free_slots == 0
    with pytest.raises(StateError):
        pool.open()
    a.position = 99
    pool.reserve(a, 1)
    with pytest.raises(StateError):
        pool.reserve(a, 2)
    pool.close(a)
    with pytest.raises(StateError):
        pool.close(a)
    assert pool.open().slot == a.slot


class CountingModel:
    """Serves without a device: the next token is a hash of everything the sequence has seen."""
    vocabulary = 50

    def __init__(self, slots):
        self.state = self
        self.slots, self.seen, self.steps = slots, {}, []

    @property
    def free_slots(self):
        return self.slots - len(self.seen)

    def open(self):
        sequence = Sequence(slot=min(set(range(self.slots)) - {s.slot for s in self.seen.values()} or {0}))
        self.seen[id(sequence)] = sequence
        sequence.history = []
        return sequence

    def close(self, sequence):
        del self.seen[id(sequence)]

    def _row(self, sequence):
        row = np.zeros(self.vocabulary, dtype=np.float32)
        row[sum((i + 1) * t for i, t in enumerate(sequence.history)) % self.vocabulary] = 1.0
        return row

    def step(self, sequence, tokens, want):
        self.steps.append(len(tokens))
        rows = []
        for place, token in enumerate(tokens):
            sequence.history.append(token)
            if place in list(want):
                rows.append(self._row(sequence))
        return np.array(rows, dtype=np.float32).reshape(len(rows), self.vocabulary)

    def decode(self, sequence, token):
        self.last = self.step(sequence, [token], [0])[0]
        return int(np.argmax(self.last))

    def logits_row(self):
        return self.last


def counted(prompt, count):
    history = list(prompt)
    for _ in range(count):
        history.append(sum((i + 1) * t for i, t in enumerate(history)) % 50)
    return history[len(prompt):]


def test_engine_schedules_portions_and_slots():
    model = CountingModel(slots=2)
    prompts = [list(range(1, 1 + n)) for n in (17, 1, 9, 4, 30)]
    engine = Engine(model, portion=8)
    assert engine.generate(prompts, max_new_tokens=5) == [counted(p, 5) for p in prompts]
    assert model.free_slots == 2 and not engine.busy
    assert max(model.steps) <= 9  # a portion, or a portion and the one token left behind it
    # while a long prompt is read, running requests keep producing
    model = CountingModel(slots=2)
    engine = Engine(model, portion=4)
    short, long = engine.submit([1, 2], 50), engine.submit(list(range(40)), 1)
    for _ in range(12):
        engine.tick()
    assert len(short.tokens) >= 5 and long.prompt_done >= 16
    engine.run()
    assert short.tokens == counted([1, 2], 50) and long.tokens == counted(list(range(40)), 1)


def test_engine_refuses_and_recovers():
    model = CountingModel(slots=1)
    engine = Engine(model)
    for prompt, count in (([], 1), ([50], 1), ([1], 0)):
        with pytest.raises(ValueError):
            engine.submit(prompt, count)
    engine.submit([1, 2], 3)
    failing = model.step
    model.step = lambda *a: (_ for _ in ()).throw(RuntimeError("device"))
    with pytest.raises(RuntimeError):
        engine.run()
    model.step = failing
    assert model.free_slots == 1 and engine.generate([[3]], 2) == [counted([3], 2)]


def test_trace_replay_over_a_host_model(tmp_path):
    model, answers = CountingModel(slots=2), []
    lines = [{"step": 0, "entries": [{"id": "a", "tokens": [1, 2, 3], "want": [0, 2]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [4], "want": []}], "end": ["a"]},
             {"step": 2, "entries": [{"id": "a", "tokens": [1], "want": [0]}], "end": ["a"]}]
    trace_replay.replay(model, io.StringIO("\n".join(map(json.dumps, lines))), str(tmp_path), answers.append)
    assert answers == ["done 0", "done 1", "done 2"] and model.free_slots == 2
    rows = np.fromfile(tmp_path / "0.f32", dtype="<f4").reshape(2, 50)
    assert rows.argmax(1).tolist() == [1, 14]
    assert not (tmp_path / "1.f32").exists()
    assert np.fromfile(tmp_path / "2.f32", dtype="<f4").argmax() == 1  # a new request of the same name


def test_sampling_of_float32_rows():
    rng = np.random.default_rng(0)
    for seed in range(1, 40):
        row = rng.standard_normal(300).astype(np.float16)
        params = sampling.Params.create(0.8, 40, 0.9, 0.02, seed)
        assert sampling.sample_f32(params, row.astype(np.float32)) == sampling.sample(params, 300, row.tobytes())
    row = np.array([0.0, 3.0, 3.0, 1.0], dtype=np.float32)
    greedy = sampling.Params.greedy()
    assert sampling.sample_f32(greedy, row) == 1 and sampling.sample_f32(greedy, row, [1]) == 2
    with pytest.raises(sampling.SamplingError):
        sampling.sample_f32(greedy, row, [4])
    with pytest.raises(sampling.SamplingError):
        sampling.sample_f32(greedy, row, [0, 1, 2, 3])


# ---- the restatement itself ----------------------------------------------------------------------------

def test_restated_attention_closed_forms():
    t, heads = 12, 2
    rng = np.random.default_rng(1)
    v = rng.standard_normal((t, 1, 3))
    q, k = np.zeros((t, heads, 4)), rng.standard_normal((t, 1, 4))
    # equal scores and a sink of weight one: the mean over the chunk's keys and one empty one
    out = hybrid_model.chunk_attention(q, k, v, 1.0, 5.0, np.zeros(heads), 5)
    for i in range(t):
        seen = range(i // 5 * 5, i + 1)
        assert np.allclose(out[i, 0], v[list(seen), 0].sum(0) / (len(seen) + 1))
    # a score far beyond the cap counts as the cap
    q[:, :, 0] = 1e6
    k[:] = 0.0
    k[0, 0, 0] = 1.0
    out = hybrid_model.chunk_attention(q, k, v, 1.0, 2.0, np.full(heads, -np.inf), None)
    weight = np.exp(2.0) / (np.exp(2.0) + 3)
    assert np.allclose(out[3, 1], weight * v[0, 0] + (1 - weight) / 3 * v[1:4, 0].sum(0))


def test_restated_recurrence_closed_form():
    """A constant input: the state is a geometric sum."""
    t, a, dt = 6, 0.7, 0.3
    x, b = np.ones((t, 1, 1)), np.ones((t, 1, 1))
    y = hybrid_model.ssm_scan(x, b, b, np.full((t, 1), dt), np.array([a]), np.array([2.0]))
    decay = np.exp(-a * dt)
    assert np.allclose(y[:, 0, 0], [dt * sum(decay ** j for j in range(i + 1)) + 2.0 for i in range(t)])


def test_restated_convolution_and_router():
    x = np.arange(1.0, 6.0)[:, None]
    assert hybrid_model.causal_conv(x, np.array([[1.0, 10.0]]), np.array([0.5]))[:, 0].tolist() == \
        [10.5, 21.5, 32.5, 43.5, 54.5]
    chosen, weights = hybrid_model.route(np.array([0.0, np.log(3.0), -1.0, 0.0]), 2)
    assert chosen.tolist() == [1, 0] and np.allclose(weights, [0.75, 0.25])


def test_restatement_is_causal_and_chunked():
    cfg = config(mamba2(mlp=dense()), attention(chunk=5, mlp=moe()))
    _, weights = make_weights(cfg, 1)
    tokens = np.random.default_rng(2).integers(0, 90, 14)
    whole = hybrid_model.forward(cfg, weights, tokens)[0]
    assert np.allclose(hybrid_model.forward(cfg, weights, tokens[:9])[0], whole[:9])
    only = config(attention(chunk=5, mlp=dense()))
    _, weights = make_weights(only, 1)
    assert np.allclose(hybrid_model.forward(only, weights, tokens[5:10])[0],
                       hybrid_model.forward(only, weights, tokens)[0][5:10])


# ---- the Koketar design --------------------------------------------------------------------------------

def test_parallel_config_reads_every_size():
    cfg = pu.config(pu.parallel(mlp=pu.dense(33, 2.5)), pu.parallel(pu.window(size=9, rotated=6, base=70.0, factor=1.5),
                                                                    pu.delta(5, 1, 7, 9, 3), 0.25, 1.75))
    parsed = LayeredConfig.parse(cfg)
    assert parsed.design is DESIGNS["Koketar"] and parsed.residual_scale == 0.7 and parsed.logit_softcap == 12.0
    first, second = parsed.layers
    assert first.mixer.left == WindowMixer(6, 2, 24, 40, 0.3, 0.0, 21, Rotation(14, 5000.0, 3.0))
    assert first.ffn == DenseFfn(33, 2, 2.5) and second.ffn is None
    assert second.mixer.right == DeltaMixer(5, 1, 7, 9, 3)
    assert (second.mixer.left_scale, second.mixer.right_scale) == (0.25, 1.75)
    assert np.allclose(second.mixer.left.rotation.frequencies, [70.0 ** (-2 * i / 6) / 1.5 for i in range(3)])
    shapes = parsed.tensor_shapes()
    assert shapes["l1.mix.right.v.conv"] == (45, 3) and shapes["l1.mix.right.a2"] == (35, None)
    assert shapes["l1.mix.left.o"] == (72, 240) and shapes["l0.mix.left.k.norm"] == (24,)
    assert "head" not in shapes and "l1.norm2" not in shapes and "l0.norm2" in shapes
    columns = JointColumns.of(second.mixer, 11, 6)
    assert columns.conv == 272 and columns.decay == 272 + 64 and columns.gate == 336 + 16 and columns.split == 360
    assert columns.total == 365
    assert model_registry.model_class({"architecture": "Koketar"}) is LayeredModel


@pytest.mark.parametrize("bad", [
    pu.config(pu.parallel(pu.window(heads=5, kv_heads=2))),
    pu.config(pu.parallel(right=pu.delta(heads=5, kv_heads=2))),
    pu.config(pu.parallel(pu.window(rotated=7))),
    pu.config(pu.parallel(pu.window(dim=8, rotated=10))),
    pu.config(pu.parallel(mlp=pu.dense(8, None))),
    pu.config(pu.parallel(mlp=moe())),
    pu.config(attention()),
    config(pu.parallel()),
])
def test_parallel_config_refuses(bad):
    with pytest.raises(ValueError):
        LayeredConfig.parse(bad)


def test_a_design_without_options_of_its_mechanisms():
    cfg = pu.config(pu.parallel(mlp=pu.dense()), softcap=None)
    left = cfg["layers"][0]["mixer"]["left"]
    del left["mask"]
    del left["rot"]["scaling"]
    parsed = LayeredConfig.parse(cfg)
    assert parsed.logit_softcap == 0.0 and parsed.layers[0].mixer.left.window == 0
    assert parsed.layers[0].mixer.left.rotation == Rotation(14, 5000.0, 1.0)


def test_ranks_come_from_the_weights(tmp_path):
    parsed = LayeredConfig.parse(pu.config(pu.parallel()))
    patterns = parsed.random_tensors(np.random.default_rng(0), rank=5)
    path = str(tmp_path / "w.safetensors")
    write_safetensors(path, patterns)
    for source in (patterns, SafetensorsFile(path)):
        tensors = _Tensors(parsed, source)
        assert tensors["l0.mix.right.a1"].shape == (5, 72) and tensors["l0.mix.right.g2"].shape == (112, 5)
    wrong = dict(patterns, **{"l0.mix.right.a2": patterns["l0.mix.right.a2"][:-1]})
    with pytest.raises(ValueError):
        _Tensors(parsed, wrong)["l0.mix.right.a2"]


def test_restated_window_and_rotation():
    t, rng = 9, np.random.default_rng(3)
    v, k = rng.standard_normal((t, 1, 3)), rng.standard_normal((t, 1, 4))
    out = parallel_model.window_attention(np.zeros((t, 2, 4)), k, v, 1.0, 4)
    for i in range(t):
        assert np.allclose(out[i, 1], v[max(0, i - 3):i + 1, 0].mean(0))
    # a rotation keeps lengths, leaves the rest alone, and makes products depend on distances
    x = rng.standard_normal((1, 1, 6)).repeat(t, axis=0)
    turned = parallel_model.rotate(x, 4, 30.0, 2.0)
    assert np.allclose(turned[:, :, 4:], x[:, :, 4:]) and np.allclose(turned[0], x[0])
    assert np.allclose((turned ** 2).sum(-1), (x ** 2).sum(-1))
    products = turned[:, 0] @ turned[:, 0].T
    assert np.allclose(products[5, 2], products[8, 5]) and not np.allclose(products[5, 2], products[5, 3])


def test_restated_delta_rule_closed_forms():
    """Without decay and with full write strength a key holds what was written to it last; a channel's decay acts on what
    its key component wrote."""
    e = np.eye(3)
    k = np.array([e[0], e[1], e[0]])[:, None]
    v = np.arange(6.0).reshape(3, 1, 2) + 1.0
    ones = np.ones((3, 1, 3))
    out = parallel_model.delta_scan(np.array([e[0], e[0], e[0] + e[1]])[:, None], k, v, ones, np.ones((3, 1)))
    assert np.allclose(out[:, 0], [v[0, 0], v[0, 0], v[2, 0] + v[1, 0]])
    decay = ones * np.array([0.5, 0.25, 1.0])
    out = parallel_model.delta_scan(np.array([e[0] + e[1]] * 3)[:, None], k[:2].repeat([1, 2], axis=0), v, decay,
                                    np.ones((3, 1)))
    assert np.allclose(out[2, 0], 0.25 * v[0, 0] + v[2, 0])


def test_restated_convolution_norms_and_feed_forward():
    x = np.arange(1.0, 6.0)[:, None]
    assert parallel_model.short_conv(x, np.array([[1.0, 10.0]]))[:, 0].tolist() == [10.0, 21.0, 32.0, 43.0, 54.0]
    assert np.allclose(parallel_model.offset_rms_norm(np.full((1, 4), 3.0), np.array([0.0, 1.0, -1.0, 0.5]), 0.0),
                       [[1.0, 2.0, 0.0, 1.5]])
    assert np.allclose(np.linalg.norm(parallel_model.unit(np.array([[3.0, 4.0]]))), 1.0)
    one = np.ones((1, 1))
    out = [parallel_model.clamped_ffn(np.array([[z]]), one, one, one, 2.0)[0, 0] for z in (-9.0, 1.0, 9.0)]
    gate = lambda g: g / (1.0 + np.exp(-1.702 * g))
    assert np.allclose(out, [gate(-9.0) * -1.0, gate(1.0) * 2.0, gate(2.0) * 3.0])


def test_restated_parallel_model_is_causal():
    cfg = pu.config(pu.parallel(pu.window(size=5), mlp=pu.dense()), pu.parallel())
    _, weights = make_weights(cfg, 1)
    tokens = np.random.default_rng(2).integers(0, 90, 14)
    whole, streams = parallel_model.forward(cfg, weights, tokens)
    part, part_streams = parallel_model.forward(cfg, weights, tokens[:9])
    assert np.allclose(part, whole[:9]) and np.allclose(part_streams, streams[:, :9])
    assert np.abs(whole).max() <= 12.0
