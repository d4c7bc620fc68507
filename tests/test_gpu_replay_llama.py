"""Token replay (ffmi_rm_replay_step) drives the LLaMA models too: logits do
not depend on how a prompt is cut, and decoding what generate() picked returns
the picks."""
import numpy as np
import pytest

import flexflow_amd as fa

pytestmark = pytest.mark.gpu

CFG = dict(num_layers=2, vocab_size=500, num_heads=2, num_kv_heads=2, hidden=128, intermediate=256,
           rms_eps=1e-6, rope_theta=10000.0)


@pytest.mark.parametrize("full", [False, True])
def test_replay_matches_generation(full):
    kw = dict(max_requests=2, max_tokens=32, max_seq_len=64, weight_seed=7, full_precision=full)
    prompt = [5, 17, 300, 42, 9, 471, 8]
    m = fa.Model(CFG, "inc", **kw)
    rm = fa.RequestManager(max_requests_per_batch=2, max_tokens_per_batch=32, max_sequence_length=64)
    seq = fa.generate(rm, m, [prompt], max_length=30)[0].output_tokens
    rm2 = fa.RequestManager(max_requests_per_batch=2, max_tokens_per_batch=32, max_sequence_length=64)
    n = len(seq) - 1
    whole = rm2.replay_step(m, [(1, seq[:n], range(n))])
    rm2.replay_end(m, 1)
    parts, at = [], 0
    for k in (3, 1, 9, 2, 1, 30):
        part = seq[at:min(at + k, n)]
        parts.append(rm2.replay_step(m, [(2, part, range(len(part))), (3, [5], [])][:1 + (at == 0)]))
        at += len(part)
    parts = np.concatenate(parts)
    assert parts.shape == whole.shape == (n, 500)
    assert np.abs(parts - whole).max() < (1e-4 if full else 2e-2) * np.abs(whole).max()
    lead = whole[np.arange(n), whole.argmax(1)] - whole[np.arange(n), seq[1:]]
    assert lead[len(prompt):].max() <= (1e-5 if full else 1e-2)
