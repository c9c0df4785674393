"""Llama on the serving engine equals its own full forward: the engine, the
cache manager and the scheduler belong to no single design."""

import pytest
import torch

pytestmark = pytest.mark.gpu


@pytest.fixture(scope="module", autouse=True)
def _groups():
    from neuronx_distributed_amd.inference import single_process_groups
    from neuronx_distributed_amd.ops import serving

    serving.ensure_built()
    single_process_groups()


def _model(window=None, dtype=torch.float32, name="tiny"):
    from neuronx_distributed_amd.models import build_model, get_config

    torch.manual_seed(0)
    return build_model("LlamaForCausalLM", get_config(
        name, sliding_window=window, max_position_embeddings=512,
        initializer_range=0.2), dtype, "cuda")


@pytest.mark.parametrize("window", [None, 50])
def test_portions_and_decoding(window):
    from neuronx_distributed_amd.inference import InferenceEngine, StepEntry

    m = _model(window)
    x = torch.randint(0, m.config.vocab_size, (1, 200), device="cuda")
    with torch.no_grad():
        want = m(x)[0].double()
    toks = x[0].tolist()
    eng = InferenceEngine(m, 512, 2)
    for cuts in ([200], [64, 3, 1, 1, 131], [150] + [1] * 50):
        out, at = [], 0
        for n in cuts:
            out.append(eng.step([StepEntry("a", toks[at:at + n], range(n))]))
            at += n
        eng.finish("a")
        err = (torch.cat(out).double() - want).abs().max() / want.abs().max()
        assert err < 2e-5, (window, cuts[:4], err.item())


def test_continuous_batch_equals_generate():
    from neuronx_distributed_amd.inference import generate, generate_ragged

    m = _model(name="test-d128")
    prompts = [torch.randint(0, 1024, (n,)).tolist() for n in (5, 70, 1, 33)]
    got = generate_ragged(m, prompts, 8, max_seqs=2, max_step_tokens=40)
    for p, g in zip(prompts, got):
        x = torch.tensor([p], device="cuda")
        assert generate(m, x, 8)[0, len(p):].tolist() == g


def test_bf16_and_table_limit():
    from neuronx_distributed_amd.inference import InferenceEngine, StepEntry

    m = _model(dtype=torch.bfloat16, name="test-d128")
    x = torch.randint(0, 1024, (1, 130), device="cuda")
    with torch.no_grad():
        want = m(x)[0].double()
    with pytest.raises(ValueError):
        InferenceEngine(m, 1024, 1, max_context=513)
    eng = InferenceEngine(m, 1024, 1)
    assert eng.cache.max_context == 512
    out = torch.cat([eng.step([StepEntry(0, x[0, :100].tolist(),
                                         range(100))])]
                    + [eng.step([StepEntry(0, [t], [0])])
                       for t in x[0, 100:].tolist()]).double()
    err = (out - want).pow(2).mean(1).sqrt() / want.pow(2).mean().sqrt()
    assert err.max() < 0.05, err.max().item()
