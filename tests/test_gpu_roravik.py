"""GPU tests of the Roravik design on the layer-list engine against the plain float64 model in tests/roravik_oracle.py: every mechanism
alone in a small model, layer by layer and through a portion and token-by-token decoding; then a model of all of them -- the stream behind
every layer run, whole prompts, decoding from the first token, portions down to one and two tokens, unequal batches, state slots and cache
blocks that are used again; tokens just inside and just outside a window, prompts and decoding, windows and blocks of every relation; one key
that decides the scores, a sink that outweighs all of them; decays at their extremes, far tokens in both kinds of state, the grouped
router alone, long decoding, greedy generation through the static batch, the scheduler and the pipeline, and bin/trace_run.
Configurations and weights are the tests' own."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from lmdeploy_amd import _ffi
from lmdeploy_amd.turbomind import layered
from tests import roravik_oracle as ro

pytestmark = pytest.mark.gpu

TOL = {'float32': 3e-5, 'bfloat16': 8e-2}
DTYPES = ['float32', 'bfloat16']


def model_folder(tmp_path, cfg, seed, name='m', change=None, rank=6):
    w = ro.random_weights(cfg, seed, rank)
    if change:
        change(w)
    folder = str(tmp_path / name)
    ro.write_checkpoint(folder, cfg, w)
    return folder, w


def engine(folder, dtype, **kw):
    args = dict(max_batch_size=4, session_len=512, cache_blocks=12, max_prefill_token_num=512, use_graph=0)
    args.update(kw)
    return layered.build_engine(folder, dtype=dtype, **args)


def row_errs(got, ref):
    d = got - ref
    d = d - d.mean(-1, keepdims=True)
    return np.sqrt((d ** 2).mean(-1)) / ref.std()


def rel_err(got, ref):
    return row_errs(got, ref).max()


def close(got, ref, dtype):
    """fp32: every row within the tolerance.  bf16: the median far inside it; every head and every sublayer is scaled to unit size, so a row
    whose result lies near zero somewhere carries more rounding: two rows of a hundred may, up to twice the tolerance"""
    e = row_errs(got, ref)
    if dtype == 'float32':
        return e.max() <= TOL[dtype]
    return np.median(e) <= TOL[dtype] / 4 and (e > TOL[dtype]).sum() <= max(1, 0.02 * len(e)) and e.max() <= 2 * TOL[dtype]


def settled_request(cfg, w, n, rng, dtype):
    """n random tokens; for bf16 runs they open with tokens whose logits the float64 model keeps when its matrices move by bf16-sized noise.  A
    state that holds ONE token answers with that token's value times query . key, and the norm behind it leaves the sign of that number:
    where it lies near zero, rounding decides"""
    head = min(n, 6)
    for _ in range(100):
        toks = rng.integers(0, cfg['vocab'], head).tolist()
        ref, worst = ro.forward(cfg, w, toks), 0.0
        for k in range(8 if dtype == 'bfloat16' else 0):
            noise = np.random.default_rng(100 + k)
            noisy = {a: b * (1 + noise.normal(0, 2.0 ** -8, b.shape)) if b.ndim == 2 else b for a, b in w.items()}
            worst = max(worst, rel_err(ro.forward(cfg, noisy, toks), ref))
        if worst <= 1.5 * TOL[dtype]:
            return toks + rng.integers(0, cfg['vocab'], n - head).tolist()
    raise AssertionError('no settled opening')


def run_cuts(eng, toks, cuts):
    """logits of every position of one request fed in portions of the given sizes"""
    s, at, rows = eng.open_session(), 0, []
    for n in cuts:
        rows.append(eng.step_tokens([(s, toks[at:at + n], list(range(n)))]))
        at += n
    eng.close_session(s)
    assert at == len(toks)
    return np.concatenate(rows)


def full_model(routed=True):
    """both mixers in several forms: grouped and ungrouped heads, sizes on and off the 8 grid, value sizes that differ from the key sizes,
    windows that cut cache blocks, rotation of a part of a head, 2 to 4 taps, shared experts smaller and larger than the routed ones, blocks
    without feed-forward, a loop of three passes over two layers.  routed=False: every expert is chosen (bf16 rounding cannot turn a choice)"""
    top = (3, 4) if routed else (8, 6)
    return ro.make_config(72, 211, [
        ro.retention_layer(3, 20, 12, [0.6, 0.95, 0.998], 3000.0, 12, ro.dense(88, 0.9)),
        ro.parallel_layer(6, 2, 16, 24, 50, 3, 12, 0.3, 9.0, 4, 500.0, 8, 0.6, 1.3,
                          ro.moe(8, top[0], 24, 4 if routed else 1, 2 if routed else 1, 20)),
        ro.retention_layer(2, 16, 40, [0.9, 0.99]),
        ro.parallel_layer(3, 3, 20, 12, 70, 2, 32, 0.25, 30.0, 2, 9000.0, 20, 1.1, 0.4, ro.dense(40, 2.0)),
        ro.parallel_layer(4, 1, 8, 16, 7, 4, 8, 0.5, 15.0, 3, mlp=ro.moe(6, top[1], 16, 1, 1, 33)),
    ], eps=1e-5, embed_scale=2.0, loop=(1, 3, 3))


RET = dict(heads=2, dim=16, vdim=16, decay=[0.8, 0.99])
PAR = dict(heads=4, kv_heads=2, dim=16, vdim=16, window=40, r_heads=2, r_dim=16)


def ret(width=48, mlp=None, eps=1e-5, loop=None, **kw):
    return lambda: ro.make_config(width, 97, [ro.retention_layer(**dict(RET, **kw), mlp=mlp)], eps=eps, loop=loop)


def par(width=48, mlp=None, eps=1e-5, loop=None, **kw):
    return lambda: ro.make_config(width, 97, [ro.parallel_layer(**dict(PAR, **kw), mlp=mlp)], eps=eps, loop=loop)


ALONE = {
    'retention': ret(),
    'retention_one_head_odd_sizes': ret(50, heads=1, dim=10, vdim=7, decay=[0.97]),
    'retention_part_of_the_rotation': ret(heads=3, dim=24, vdim=40, decay=[0.5, 0.9, 0.999], rot_dims=6, base=50.0),
    'retention_no_rotation': ret(rot_dims=0),
    'retention_head_128': ret(64, dim=128, vdim=128, base=1e6),
    'retention_head_256_values_72': ret(heads=1, dim=256, vdim=72, decay=[0.995]),
    'retention_values_150': ret(heads=2, dim=33, vdim=150, rot_dims=32),
    'retention_decays_at_their_ends': ret(heads=4, dim=8, vdim=8, decay=[0.0, 1.0, 1e-6, 0.9999]),
    'parallel': par(),
    'parallel_left_alone': par(right_scale=0.0),
    'parallel_right_alone': par(left_scale=0.0),
    'parallel_window_1_one_tap': par(window=1, conv=1),
    'parallel_window_64_two_taps': par(window=64, conv=2),
    'parallel_window_beyond_the_prompt_eight_taps': par(window=1000, conv=8),
    'parallel_sixteen_taps': par(conv=16),
    'parallel_odd_sizes': par(51, heads=3, kv_heads=1, dim=10, vdim=7, window=33, r_heads=3, r_dim=5, rot_dims=4),
    'parallel_everything_equal': par(32, heads=1, kv_heads=1, dim=32, vdim=32, window=32, r_heads=1, r_dim=32, scale=1.0, left_scale=1.0, right_scale=1.0),
    'parallel_no_rotation_tight_cap': par(rot_dims=0, softcap=1.5, scale=1.0),
    'parallel_24_heads': par(64, heads=24, kv_heads=8, dim=8, vdim=8, r_heads=9, r_dim=8),
    'parallel_head_128': par(64, heads=2, kv_heads=1, dim=128, vdim=128, window=100, r_heads=1, r_dim=128),
    'parallel_head_256': par(heads=1, kv_heads=1, dim=256, vdim=200, window=90, r_heads=1, r_dim=256),
    'parallel_state_head_50': par(r_heads=3, r_dim=50),
    'dense_tight_limit': ret(mlp=ro.dense(100, 0.2)),
    'dense_wide_limit': par(mlp=ro.dense(3000, 50.0)),
    'dense_of_one': ret(mlp=ro.dense(1, 1.0)),
    'experts_one_group': ret(mlp=ro.moe(8, 2, 24, 1, 1, 24)),
    'experts_of_groups_of_one': ret(mlp=ro.moe(6, 2, 24, 6, 3, 40)),
    'experts_top_1_shared_larger': par(mlp=ro.moe(12, 1, 20, 3, 1, 52)),
    'experts_all_kept': par(mlp=ro.moe(12, 5, 20, 4, 4, 8)),
    'experts_every_one': ret(mlp=ro.moe(5, 5, 16, 1, 1, 16)),
    'experts_eighty_in_ten_groups': ret(mlp=ro.moe(80, 6, 8, 10, 3, 8)),
    'experts_three_hundred': ret(32, mlp=ro.moe(300, 4, 4, 50, 2, 4)),
    'loop_whole_model': ret(loop=(0, 1, 3)),
    'loop_once': par(loop=(0, 1, 1)),
    'loop_at_the_start': lambda: ro.make_config(40, 97, [ro.parallel_layer(**PAR, mlp=ro.dense(24)), ro.retention_layer(**RET)], loop=(0, 1, 4)),
    'loop_at_the_end': lambda: ro.make_config(40, 97, [ro.retention_layer(**RET), ro.retention_layer(**RET), ro.parallel_layer(**PAR)], loop=(1, 3, 2)),
    'large_eps': par(eps=0.3, mlp=ro.dense(40)),
    'width_1100': par(1100, mlp=ro.dense(40)),
    'width_5000': ret(5000, mlp=ro.dense(24)),
    'width_9000': par(9000, mlp=ro.dense(24)),
}
# a result of one value, or a head that holds a single key times its product with the query, may lie next to zero, where the norm behind it
# scales rounding up to the size of a full result: a few rows, in bf16 only
FEW = {'dense_of_one', 'retention_decays_at_their_ends'}


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('name', list(ALONE))
def test_each_mechanism_alone(cuda, tmp_path, dtype, name):
    cfg = ALONE[name]()
    toks = np.random.default_rng(1).integers(0, 97, 150).tolist()
    folder, w = model_folder(tmp_path, cfg, 3, rank=40 if '128' in name else 3)
    gaps = []
    ref, trail = ro.forward(cfg, w, toks, True, gaps)
    # rows whose closest expert choice bf16 rounding could turn (another function of the token from there on) are left out; fp32 keeps all
    clear = np.ones(len(toks), bool) if dtype == 'float32' or not gaps else np.min(gaps, axis=0) > 0.03
    # ('all' experts are always clear; what is left out must stay a part)
    assert clear.mean() > (0.1 if name.endswith('hundred') or 'eighty' in name else 0.3), clear.mean()
    eng = engine(folder, dtype)
    for n in range(1, len(trail) + 1):
        eng.stop_after(n)
        s = eng.open_session()
        eng.step_tokens([(s, toks, [])])
        got = eng.fetch_residual(len(toks))
        eng.close_session(s)
        err = np.abs(got - trail[n - 1])[clear].max(-1) / np.abs(trail[n - 1]).max()
        assert (err > TOL[dtype] * 3).sum() <= (3 if dtype == 'bfloat16' and name in FEW else 0), (n, err.max())
    eng.stop_after(-1)
    for cuts in ([75] + [1] * 75, [2, 1, 15, 17, 64, 51]):        # the same through cache and state
        errs = row_errs(run_cuts(eng, toks, cuts), ref)[clear]
        assert (errs > TOL[dtype]).sum() <= (3 if dtype == 'bfloat16' and name in FEW else 0), (cuts[:3], np.sort(errs)[-5:])
    eng.close()


@pytest.mark.parametrize('dtype', DTYPES)
def test_engine_layers_and_whole_prompt(cuda, tmp_path, dtype):
    cfg = full_model(dtype == 'float32')
    folder, w = model_folder(tmp_path, cfg, 0)
    eng = engine(folder, dtype)
    toks = np.random.default_rng(1).integers(0, cfg['vocab'], 150).tolist()
    ref, trail = ro.forward(cfg, w, toks, True)
    assert len(trail) == 9
    for n in range(1, len(trail) + 1):                            # the residual stream behind every layer run
        eng.stop_after(n)
        s = eng.open_session()
        eng.step_tokens([(s, toks[:70], [])])
        got = eng.fetch_residual(70)
        eng.close_session(s)
        assert np.abs(got - trail[n - 1][:70]).max() <= TOL[dtype] * 3 * np.abs(trail[n - 1]).max(), n
    eng.stop_after(-1)
    assert close(run_cuts(eng, toks, [150]), ref, dtype)
    eng.close()


@pytest.mark.parametrize('dtype', DTYPES)
def test_engine_portions_decoding_batches_and_reuse(cuda, tmp_path, dtype):
    """every way of cutting the same requests gives the oracle's logits: token by token from the first token on, portions down to one and
    two tokens (shorter than the convolutions' reach) that start and end inside blocks, windows and chunks, unequal requests in one forward,
    and sessions that come and go in a pool that holds only what is live -- cache blocks and state slots are used again with other
    requests' keys, convolution inputs, previous tokens and states still in them"""
    cfg = full_model(dtype == 'float32')
    folder, w = model_folder(tmp_path, cfg, 1)
    rng = np.random.default_rng(2)
    reqs = [settled_request(cfg, w, n, rng, dtype) for n in (200, 131, 65, 1, 23)]
    refs = [ro.forward(cfg, w, t) for t in reqs]
    eng = engine(folder, dtype, cache_blocks=9)
    assert close(run_cuts(eng, reqs[1], [1] * 131), refs[1], dtype)
    for cuts in ([2, 1, 2, 58, 2, 64, 3, 30, 2] + [1] * 36, [2] * 100, [17, 16, 15, 33, 32, 31, 7, 49], [63, 2, 62, 2, 71]):
        assert close(run_cuts(eng, reqs[0], cuts), refs[0], dtype), cuts
    plan = [[(0, 60)], [(0, 4), (1, 64), (3, 1)], [(0, 1), (1, 2), (2, 33)], [(1, 1), (2, 2), (4, 23)], [(0, 64), (2, 30)],
            [(0, 1), (1, 64)], [(0, 70)]]
    sess, at, got = {}, [0] * 5, [[] for _ in reqs]
    for step in plan:
        entries = []
        for r, n in step:
            if r not in sess:
                sess[r] = eng.open_session()
            entries.append((sess[r], reqs[r][at[r]:at[r] + n], list(range(n))))
        out, k = eng.step_tokens(entries), 0
        for r, n in step:
            got[r].append(out[k:k + n])
            k += n
            at[r] += n
            if at[r] == len(reqs[r]):
                eng.close_session(sess.pop(r))
    assert at == [200, 131, 65, 1, 23] and not sess
    for r in range(5):
        assert close(np.concatenate(got[r]), refs[r], dtype), r
    a, b = eng.open_session(), eng.open_session()                 # the pool is bounded: a step that cannot fit is refused and changes nothing
    eng.step_tokens([(a, reqs[0][:200], []), (b, reqs[1][:131], [])])
    with pytest.raises(_ffi.TmError):
        eng.step_tokens([(b, reqs[1][:131], [])])
    eng.close_session(a)
    out = eng.step_tokens([(b, [5], [0])])
    assert close(out, ro.forward(cfg, w, reqs[1] + [5])[-1:], dtype)
    eng.close_session(b)
    eng.close()


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('window', [2, 50, 64, 65, 100, 128])
def test_tokens_just_inside_and_just_outside_a_window(cuda, tmp_path, dtype, window):
    """one layer whose only way back in time is the window (one tap, the right mixer weighing zero): a token whose key answers every query
    louder than all others, put at the window's last position, moves the row's logits; one position earlier it leaves them as they were --
    rows inside blocks and on block borders, as part of a prompt, at the end of a portion of two, and decoded"""
    cfg = ro.make_config(48, 61, [ro.parallel_layer(**dict(PAR, window=window, conv=1, right_scale=0.0, rot_dims=8))])

    def loud(w):            # channel 0 is in every token and in every query, channel 1 in token 60 and in every key: they meet behind the rotated part
        w['embed'][:, 0], w['embed'][:, 1], w['embed'][60, 1] = 1.0, 0.0, 1.0
        for t, ch in (('q', 0), ('k', 1)):
            a = w['l0.mix.left.' + t].reshape(-1, 16, 48)
            a[:, :, ch] = 0.0
            a[:, 8:, ch] = 2.0
    folder, w = model_folder(tmp_path, cfg, 21, change=loud)
    eng = engine(folder, dtype)
    rng = np.random.default_rng(5)
    lim = TOL[dtype] if dtype == 'float32' else 0.15
    moved = []
    for pos in (63, 64, 129, 191, 192, 300):
        base = rng.integers(0, 60, pos + 1).tolist()
        ref0 = ro.forward(cfg, w, base)[-1]
        for back in (window - 1, window):
            j = pos - back
            if j < 0:
                continue
            toks = list(base)
            toks[j] = 60
            ref = ro.forward(cfg, w, toks)[-1]
            if back == window:
                assert np.abs(ref - ref0).max() < 1e-9
            else:
                moved.append(np.abs(ref - ref0).max() / ref0.std())
            whole = run_cuts(eng, toks, [pos + 1])[-1:]
            split = run_cuts(eng, toks, [pos - 1, 2])[-1:]
            dec = run_cuts(eng, toks, [pos, 1])[-1:]
            for got in (whole, split, dec):
                assert rel_err(got, ref[None]) <= lim, (pos, back)
            if back == window:      # exactly the logits of the prompt without it, whatever lies there
                assert np.array_equal(dec, run_cuts(eng, base, [pos, 1])[-1:]) and np.array_equal(whole, run_cuts(eng, base, [pos + 1])[-1:])
    assert min(moved) > 1.0           # (in units of the logits' spread)
    eng.close()


@pytest.mark.parametrize('dtype', DTYPES)
def test_single_keys_and_sinks_that_decide(cuda, tmp_path, dtype):
    """a wide window and scores far apart: the last row's logits follow ONE key wherever it lies -- first token, block borders, far back, the
    neighbour -- in a prompt and in decoding; and sinks from one that never matters to one that takes all weight"""
    rng = np.random.default_rng(5)
    worst = 0.0
    for si, sink in enumerate((-20.0, 0.0, 3.0, 60.0)):
        cfg = ro.make_config(48, 61, [ro.parallel_layer(**dict(PAR, window=1000, conv=2, scale=1.5, softcap=40.0, right_scale=0.3))])
        folder, w = model_folder(tmp_path, cfg, 21, 'm%d' % si, lambda w: w.update({'l0.mix.left.sink': np.full(4, sink)}))
        eng = engine(folder, dtype)
        for last in (63, 64, 130, 300):
            base = rng.integers(0, 60, last + 1).tolist()
            ref0 = ro.forward(cfg, w, base)[-1]
            for j in sorted({0, 63, 64, 65, 128, last - 1} & set(range(last))):
                toks = list(base)
                toks[j] = 60
                ref = ro.forward(cfg, w, toks)[-1]
                moved = np.abs(ref - ref0).max() / ref.std()
                worst = max(worst, moved)
                whole, dec = run_cuts(eng, toks, [last + 1])[-1:], run_cuts(eng, toks, [last, 1])[-1:]
                lim = TOL[dtype] if dtype == 'float32' else 0.15      # (scores of +-10 rounded to bf16 operands)
                assert rel_err(whole, ref[None]) <= lim and rel_err(dec, ref[None]) <= lim, (sink, last, j)
                if dtype == 'float32':
                    assert abs(np.abs(whole[0] - ref0).max() / ref.std() - moved) <= 3e-4, (sink, last, j)
        eng.close()
    assert worst > 0.2


def _decays(name):
    def change(w):
        b = w['l0.mix.right.w0']
        if name == 'hold':           # within 1e-3 of one: a token lives for hundreds of steps
            w['l0.mix.right.w0'] = ro.bf16_round(b * 0 - 8.0)
        elif name == 'drop':         # exp(-exp(4)): a chunk's running products underflow at once
            w['l0.mix.right.w0'] = ro.bf16_round(b * 0 + 4.0)
        elif name == 'mixed':        # channels that drop beside channels that hold
            w['l0.mix.right.w0'] = ro.bf16_round(np.where(np.arange(len(b)) % 2, 4.0, -9.0))
        elif name == 'overflow':     # exp(30) in the exponent: a decay of exactly zero
            w['l0.mix.right.w0'] = ro.bf16_round(b * 0 + 30.0)
    return change


@pytest.mark.parametrize('dtype', DTYPES)
@pytest.mark.parametrize('name', ['hold', 'drop', 'mixed', 'overflow'])
@pytest.mark.parametrize('head', [(2, 20), (1, 64)])
def test_channel_decays_at_their_extremes(cuda, tmp_path, dtype, name, head):
    cfg = ro.make_config(32, 53, [ro.parallel_layer(**dict(PAR, r_heads=head[0], r_dim=head[1], left_scale=0.1))])
    folder, w = model_folder(tmp_path, cfg, 6, change=_decays(name))
    toks = np.random.default_rng(8).integers(0, 53, 230).tolist()
    ref = ro.forward(cfg, w, toks)
    eng = engine(folder, dtype)
    for cuts in ([230], [1] * 40 + [190], [100] + [1] * 130, [15, 17, 2, 64, 132]):
        assert rel_err(run_cuts(eng, toks, cuts), ref) <= TOL[dtype], (cuts[:3], len(cuts))
    eng.close()


@pytest.mark.parametrize('kind', ['retention', 'time mixer'])
def test_state_of_a_far_token_survives_hundreds_of_steps(cuda, tmp_path, kind):
    """moving one token 300 positions back moves the last logits through the state alone, in one portion and when everything behind the first
    portion is decoded token by token"""
    if kind == 'retention':
        cfg, change = ro.make_config(32, 53, [ro.retention_layer(1, 16, 16, [0.999])]), None
    else:
        cfg, change = ro.make_config(32, 53, [ro.parallel_layer(**dict(PAR, window=4, r_heads=1, r_dim=16, left_scale=0.0))]), _decays('hold')
    folder, w = model_folder(tmp_path, cfg, 6, change=change)
    rng = np.random.default_rng(8)
    a = rng.integers(0, 53, 330).tolist()
    b = list(a)
    b[20] = (a[20] + 17) % 53
    ra, rb = ro.forward(cfg, w, a)[-1], ro.forward(cfg, w, b)[-1]
    assert np.abs(ra - rb).max() > 50 * 3e-5 * ra.std()           # the far token matters far more than the tolerance
    eng = engine(folder, 'float32')
    for toks, ref in ((a, ra), (b, rb)):
        for cuts in ([330], [25] + [1] * 305):
            assert rel_err(run_cuts(eng, toks, cuts)[-1:], ref[None]) <= 3e-5
    eng.close()


@pytest.mark.parametrize('dtype', DTYPES)
def test_engine_long_decoding(cuda, tmp_path, dtype):
    """420 tokens, the last 320 one at a time, far beyond the narrow window and with the wide one's keys split over several workgroups
    (session_len 1024 -> 4 splits)"""
    cfg = ro.make_config(64, 97, [ro.parallel_layer(**dict(PAR, window=30, conv=4), mlp=ro.dense(72)), ro.retention_layer(2, 12, 24, [0.7, 0.999]),
                                  ro.parallel_layer(**dict(PAR, heads=20, kv_heads=1, dim=16, window=350))], loop=(1, 3, 2))
    folder, w = model_folder(tmp_path, cfg, 4)
    toks = np.random.default_rng(3).integers(0, 97, 420).tolist()
    ref = ro.forward(cfg, w, toks)
    eng = engine(folder, dtype, session_len=1024, cache_blocks=17, max_prefill_token_num=256)
    assert close(run_cuts(eng, toks, [100] + [1] * 320), ref, dtype)
    eng.close()


@pytest.mark.parametrize('dtype', DTYPES)
def test_clamps_and_caps_that_bind(cuda, tmp_path, dtype):
    """weights that drive gate and up far beyond their bound on both sides, scores into their cap and logits into theirs"""
    cfg = ro.make_config(40, 97, [ro.parallel_layer(**dict(PAR, softcap=2.0, scale=2.0), mlp=ro.dense(60, 0.7)),
                                  ro.retention_layer(**RET, mlp=ro.dense(44, 3.0))], logit_softcap=3.0)

    def big(w):
        for k in ('l0.mlp.gate', 'l0.mlp.up', 'l1.mlp.gate', 'l1.mlp.up'):
            w[k] = ro.bf16_round(w[k] * 4.0)
    folder, w = model_folder(tmp_path, cfg, 9, change=big)
    toks = np.random.default_rng(2).integers(0, 97, 90).tolist()
    ref, trail = ro.forward(cfg, w, toks, True)
    assert np.abs(ref).max() > 2.5
    eng = engine(folder, dtype)
    for cuts in ([90], [33] + [1] * 57):
        assert rel_err(run_cuts(eng, toks, cuts), ref) <= TOL[dtype]
    eng.close()


def _greedy(cfg, w, prompt, n_new):
    toks, margins = list(prompt), []
    for _ in range(n_new):
        lg = ro.forward(cfg, w, toks)[-1]
        top = np.sort(lg)[-2:]
        margins.append((top[1] - top[0]) / lg.std())
        toks.append(int(np.argmax(lg)))
    return toks[len(prompt):], margins


def _check_greedy(cfg, w, prompt, toks, min_margin=2e-2):     # (the sampler reads fp16 logits rows)
    ref, margins = _greedy(cfg, w, prompt, len(toks))
    for i, (a, b, m) in enumerate(zip(toks, ref, margins)):
        if m < min_margin:
            return          # a near-tie: from here on the two may legitimately part
        assert int(a) == b, (i, toks, ref)


def test_greedy_generation_static_batch_and_scheduler(cuda, tmp_path):
    cfg = full_model()
    folder, w = model_folder(tmp_path, cfg, 2)
    rng = np.random.default_rng(6)
    prompts = [rng.integers(0, cfg['vocab'], n).tolist() for n in (70, 3, 129, 40, 64, 9)]
    eng = engine(folder, 'float32', max_batch_size=3, session_len=256, cache_blocks=13, max_prefill_token_num=128, use_graph=1)
    eng.prefill(prompts[:3], max_new_tokens=12)                   # static batch: chunked prefill + the captured decode step
    eng.decode(11)
    toks = eng.fetch()
    eng.release()
    for p, t in zip(prompts[:3], toks):
        _check_greedy(cfg, w, p, t.tolist())
    ids = [eng.submit(p, 10) for p in prompts]                    # continuous batching: six requests through three slots
    for _ in range(200):
        na, nw = eng.step()
        if na == 0 and nw == 0:
            break
    for p, rid in zip(prompts, ids):
        status, out = eng.poll(rid)
        assert status == 7 and len(out) == 10
        _check_greedy(cfg, w, p, out.tolist())
    eng.release()
    eng.close()


def test_pipeline_serves_a_checkpoint_folder(cuda, tmp_path):
    from lmdeploy_amd import GenerationConfig, TurbomindEngineConfig, pipeline
    cfg = full_model(False)
    folder, w = model_folder(tmp_path, cfg, 3)
    prompts = [np.random.default_rng(7).integers(0, cfg['vocab'], n).tolist() for n in (33, 5)]
    with pipeline(folder, backend_config=TurbomindEngineConfig(dtype='bfloat16', session_len=128, max_batch_size=2)) as pipe:
        outs = pipe(prompts, gen_config=GenerationConfig(max_new_tokens=8, ignore_eos=True))
        for p, r in zip(prompts, outs):
            assert len(r.token_ids) == 8
            _check_greedy(cfg, w, p, r.token_ids, min_margin=0.15)
        sampled = pipe(prompts, gen_config=GenerationConfig(max_new_tokens=6, ignore_eos=True, do_sample=True, top_k=5, temperature=0.8,
                                                            random_seed=11))
        assert all(len(r.token_ids) == 6 and all(0 <= t < cfg['vocab'] for t in r.token_ids) for r in sampled)


def test_captured_decode_step_equals_the_eager_one(cuda, tmp_path):
    """the decode step as a hipGraph, replayed many times, against the same engine without graphs: the same tokens, bf16, routed experts with
    a shared one inside the batched products"""
    cfg = full_model()
    folder, w = model_folder(tmp_path, cfg, 5)
    rng = np.random.default_rng(6)
    prompts = [rng.integers(0, cfg['vocab'], n).tolist() for n in (70, 3, 129)]
    outs = []
    for graph in (0, 1):
        eng = engine(folder, 'bfloat16', max_batch_size=3, session_len=256, cache_blocks=13, use_graph=graph)
        eng.prefill(prompts, max_new_tokens=40)
        for _ in range(3):                                        # replays with synchronizations between them
            eng.decode(13)
            eng.sync()
        outs.append([t.tolist() for t in eng.fetch()])
        eng.release()
        eng.close()
    assert outs[0] == outs[1]


def test_trace_run_replays_a_schedule(cuda, tmp_path):
    """bin/trace_run end to end, both number formats: a width off the 8 grid, five requests in shared steps, a request that pauses, pool of
    640 tokens"""
    rng = np.random.default_rng(0)
    plan = [[('a', 100)], [('a', 3), ('b', 64), ('c', 1)], [('a', 1), ('b', 2), ('d', 65)], [('a', 64), ('b', 1), ('d', 1), ('e', 2)],
            [('a', 2), ('b', 3), ('d', 63), ('e', 38)], [('a', 130)]]
    cfg = ro.make_config(100, 333, [ro.parallel_layer(5, 1, 12, 24, 90, 3, 20, 0.35, 25.0, 2, 700.0, 8, mlp=ro.dense(72)),
                                    ro.retention_layer(3, 20, 24, [0.9, 0.99, 0.5], mlp=ro.moe(4, 4, 24, 1, 1, 40)),
                                    ro.parallel_layer(4, 4, 24, 8, 33, 2, 10, conv=4)], embed_scale=1.5, loop=(0, 2, 2))
    folder, w = model_folder(tmp_path, cfg, 11, 'model')
    reqs = {n: settled_request(cfg, w, k, rng, 'bfloat16') for n, k in (('a', 300), ('b', 70), ('c', 1), ('d', 129), ('e', 40))}
    at, steps, rows = {n: 0 for n in reqs}, [], []
    for i, st_ in enumerate(plan):
        ent, end, rr = [], [], []
        for n, k in st_:
            ent.append({'id': n, 'tokens': reqs[n][at[n]:at[n] + k], 'want': list(range(0, k, 2))})
            rr += [(n, at[n] + j) for j in range(0, k, 2)]
            at[n] += k
            if at[n] == len(reqs[n]):
                end.append(n)
        steps.append(json.dumps({'step': i, 'entries': ent, 'end': end}))
        rows.append(rr)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    ref = {n: ro.forward(cfg, w, t) for n, t in reqs.items()}
    for dtype in DTYPES:
        out = str(tmp_path / dtype)
        p = subprocess.run([sys.executable, os.path.join(root, 'bin', 'trace_run'), '--model', folder, '--dtype', dtype, '--out', out,
                            '--max-tokens', '640'], input='\n'.join(steps) + '\n', text=True, capture_output=True, timeout=100)
        assert p.returncode == 0, p.stderr[-2000:]
        assert [l for l in p.stdout.split('\n') if l.startswith('done')] == ['done %d' % i for i in range(len(plan))]
        for i, rr in enumerate(rows):
            got = np.fromfile(os.path.join(out, '%d.f32' % i), '<f4').reshape(len(rr), -1)
            assert close(got, np.stack([ref[n][j] for n, j in rr]), dtype), (dtype, i)
