"""Scheduling over a paged cache, on the CPU with the hash test double: its
contexts are read through the page tables, so a page handed to two requests or
lost on the way changes a token."""
import pytest

import flexflow_amd as fa

VOCAB = 997


def prompts(n, seed=1):
    out, x = [], seed
    for i in range(n):
        p = []
        for _ in range(3 + (7 * i) % 29):
            x = (x * 1103515245 + 12345) % (1 << 31)
            p.append(x % VOCAB)
        out.append(p)
    return out


def serve(pool, ps, length=40, slots=4, mtb=16):
    rm = fa.RequestManager(max_requests_per_batch=slots, max_tokens_per_batch=mtb,
                           max_spec_tree_token_num=0, max_sequence_length=64)
    m = fa.HashModel(VOCAB, "inc", max_requests=slots, max_seq_len=64, max_tree_tokens=0, pool=pool)
    res = fa.generate(rm, m, ps, max_length=length)
    return [r.output_tokens for r in res], rm.stats(), m


@pytest.mark.parametrize("pages,page", [(64, 4), (16, 16), (11, 4), (3, 16)])
def test_generation_does_not_depend_on_the_pool(pages, page):
    ps = prompts(9)
    want, _, _ = serve(None, ps)
    got, _, m = serve((pages, page), ps)
    assert got == want
    assert m.free_pages() == pages  # every page came back


def test_small_pool_serves_fewer_requests_at_once():
    ps = prompts(6)
    _, wide, _ = serve((64, 8), ps)
    _, narrow, _ = serve((5, 8), ps)  # one 40-token request at a time
    assert narrow.llm_steps > 2 * wide.llm_steps


def test_a_request_larger_than_the_pool_is_an_error():
    with pytest.raises(fa.ffmi.FFMIError):
        serve((4, 8), prompts(1))


def replay_setup(pages=8, page=8, slots=3, mtb=7):
    rm = fa.RequestManager(max_requests_per_batch=slots, max_tokens_per_batch=mtb,
                           max_spec_tree_token_num=0, max_sequence_length=64)
    return rm, fa.HashModel(VOCAB, "inc", max_requests=slots, max_seq_len=64, max_tree_tokens=0,
                            pool=(pages, page))


def picks(logits):
    return [int(r.argmax()) for r in logits]


def test_replay_portions_and_batches():
    a, b = prompts(20)[3][:10] + prompts(20)[4], prompts(20)[5]
    rm, m = replay_setup()
    whole = picks(rm.replay_step(m, [(1, a, range(len(a)))]))  # more tokens than one batch holds
    rm.replay_end(m, 1)
    other = picks(rm.replay_step(m, [(2, b, range(len(b)))]))
    rm.replay_end(m, 2)
    assert m.free_pages() == 8
    got_a, got_b, ia, ib = [], [], 0, 0
    for n, k in [(2, 3), (9, 1), (1, 8), (30, 30)]:
        ta, tb = a[ia:ia + n], b[ib:ib + k]
        want_b = [i for i in range(len(tb)) if i % 2 == 0]
        out = picks(rm.replay_step(m, [(8, ta, range(len(ta))), (9, tb, want_b)]))
        got_a += out[:len(ta)]
        got_b += zip([ib + i for i in want_b], out[len(ta):])
        ia, ib = ia + len(ta), ib + len(tb)
    assert got_a == whole
    assert all(other[i] == t for i, t in got_b)
    rm.replay_end(m, 8)
    rm.replay_end(m, 9)
    assert m.free_pages() == 8


def test_replay_returns_the_order_asked_for():
    rm, m = replay_setup()
    toks = prompts(3)[2]
    ref = picks(rm.replay_step(m, [(1, toks, range(len(toks)))]))
    got = picks(rm.replay_step(m, [(2, toks, [4, 0, 4, 2]), (3, toks[:2], [1])]))
    assert got == [ref[4], ref[0], ref[4], ref[2], ref[1]]
    assert len(rm.replay_step(m, [(2, [5], [])])) == 0


def test_replay_slots_and_pages_run_out_and_come_back():
    rm, m = replay_setup(pages=4, page=8, slots=2)
    rm.replay_step(m, [(1, [5] * 16, []), (2, [6] * 9, [])])
    with pytest.raises(fa.ffmi.FFMIError):  # no third slot
        rm.replay_step(m, [(3, [7], [])])
    rm.replay_end(m, 1)
    rm.replay_step(m, [(3, [7] * 16, [])])
    with pytest.raises(fa.ffmi.FFMIError):  # no fifth page
        rm.replay_step(m, [(3, [7], [])])
    with pytest.raises(fa.ffmi.FFMIError):  # not live
        rm.replay_end(m, 1)


def test_replay_rejects_bad_entries():
    rm, m = replay_setup()
    for entries in ([(1, [5, 6], [2])], [(1, [5], [-1])], [(1, [5], []), (1, [6], [])]):
        with pytest.raises(fa.ffmi.FFMIError):
            rm.replay_step(m, entries)
