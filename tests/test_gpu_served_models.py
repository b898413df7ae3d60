"""The W4A16 transformer through the same registry, engine and command line as the layered decoders."""
import json

import numpy as np
import pytest

from llmopt_amd import cli, model_registry
from llmopt_amd.decode_step import DecodeConfig, DecodeStep, random_weights
from llmopt_amd.engine import Engine
from llmopt_amd.prefill_step import PrefillStep
from llmopt_amd.w4a16_model import W4a16Model, archive_tensors
from llmopt_amd.weight_archive import write_archive

pytestmark = pytest.mark.gpu
CONFIG = DecodeConfig(hidden=256, q_heads=4, kv_heads=2, head_dim=64, mlp=512, layers=3, vocabulary=1000)


@pytest.fixture(scope="module")
def folder(tmp_path_factory):
    path = tmp_path_factory.mktemp("w4a16")
    weights = random_weights(CONFIG, np.random.default_rng(3))
    write_archive(str(path / "weights.llmopt"), archive_tensors(weights))
    config = {"architecture": "W4A16Transformer", "hidden": 256, "q_heads": 4, "kv_heads": 2, "head_dim": 64,
              "mlp": 512, "layers": 3, "vocabulary": 1000}
    (path / "config.json").write_text(json.dumps(config))
    return path, weights


def generate_by_steps(runtime, weights, prompt, count, capacity=128):
    """Prefill and decode steps driven by hand."""
    pool = runtime.create_buffer(capacity * CONFIG.token_stride)
    slots = np.arange(capacity + 1, dtype=np.uint32)
    device_slots = runtime.buffer_of_bytes(slots)
    n = len(prompt)
    tokens = [PrefillStep(runtime, CONFIG, weights, n, pool, device_slots).run(prompt)]
    step = DecodeStep(runtime, CONFIG, weights, 1, pool, device_slots, [0], [n], [n], [n], max_context=capacity,
                      slots_host=slots)
    for i in range(count - 1):
        if i:
            step.advance()
        tokens.append(int(step.run([tokens[-1]])[0]))
    return tokens


def test_engine_gives_the_tokens_of_the_steps(folder):
    path, weights = folder
    model = model_registry.load_model(str(path), slots=2, max_context=128)
    assert isinstance(model, W4a16Model)
    rng = np.random.default_rng(4)
    prompts = [rng.integers(0, 1000, n).tolist() for n in (17, 40, 5)]
    got = Engine(model).generate(prompts, max_new_tokens=8)
    assert got == [generate_by_steps(model.runtime, weights, p, 8) for p in prompts]
    assert model.state.free_slots == 2


def test_logits_of_a_step(folder):
    path, _ = folder
    model = model_registry.load_model(str(path), slots=2, max_context=64)
    tokens = np.random.default_rng(5).integers(0, 1000, 12).tolist()
    one, two = model.open(), model.open()
    whole = model.step(one, tokens, [0, 5, 11])
    decoded = np.concatenate([model.step(two, [t], [0]) for t in tokens])
    scale = np.sqrt(np.mean(whole ** 2))
    # decoding reads quantised keys and values, the prefill the fresh ones
    assert np.sqrt(np.mean((whole - decoded[[0, 5, 11]]) ** 2)) < 0.05 * scale
    with pytest.raises(ValueError):
        model.step(one, [1000])
    with pytest.raises(ValueError):
        model_registry.load_model(str(path), activations="float32")


def test_command_line(folder, capsys):
    path, weights = folder
    prompt = [3, 14, 159, 26]
    assert cli.main(["generate", "--model", str(path), "--max-new-tokens", "4", "--max-context", "64", "--slots", "1",
                     "--prompt", " ".join(map(str, prompt))]) == 0
    runtime = model_registry.Runtime()
    assert [int(t) for t in capsys.readouterr().out.split()] == generate_by_steps(runtime, weights, prompt, 4)
    assert cli.main(["models"]) == 0
    assert capsys.readouterr().out.split() == ["Barovik", "Koketar", "W4A16Transformer"]
