"""Host tests of the Roravik design: the config reader's mapping of every constant and what it refuses, hand cases of the float64 model's
mechanisms (tests/roravik_oracle.py), and that the tests' own model shows a fault in each of them."""
import copy
import math

import numpy as np
import pytest

from lmdeploy_amd.turbomind import layered
from tests import roravik_oracle as ro


def _cfg():
    return ro.make_config(44, 103, [
        ro.retention_layer(3, 10, 7, [0.5, 0.9, 0.99], 5000.0, 6, ro.dense(30, 0.8)),
        ro.parallel_layer(6, 3, 12, 9, 37, 2, 11, 0.3, 17.0, 4, 700.0, 8, 0.6, 1.4, ro.moe(12, 2, 20, 4, 2, 26)),
        ro.parallel_layer(2, 2, 8, 8, 5, 1, 6),
        ro.retention_layer(1, 4, 4, [0.7], mlp=ro.moe(6, 3, 9, 3, 3, 5)),
    ], eps=1e-6, embed_scale=3.5, logit_softcap=9.0, loop=(1, 3, 3))


def test_reader_maps_every_constant(tmp_path):
    cfg = _cfg()
    w = ro.random_weights(cfg, 0, decay_rank=5)
    ro.write_checkpoint(str(tmp_path), cfg, w)
    assert layered.is_layered(str(tmp_path))
    c = layered.read_layered_config(str(tmp_path))
    assert (c.arch, c.width, c.vocab, c.embed_scale, c.logit_softcap) == ('Roravik', 44, 103, 3.5, 9.0)
    assert abs(c.norm_eps - 1e-6) < 1e-12 and c.norm_offset == 1.0 and c.tied_head and c.loop_add and c.loop_times == 0 and not c.final_layer_norm
    assert len(c.layers) == 8 and c.names == ['l0.', 'l1.', 'l2.', 'l1.', 'l2.', 'l1.', 'l2.', 'l3.']
    assert [s.weights_of for s in c.layers] == [-1, -1, -1, 1, 2, 1, 2, -1]
    assert [s.loop_pass for s in c.layers] == [-1, 0, -1, 1, -1, 2, -1, -1]
    assert all(s.both_norms and not s.post_norm and not s.pre_norm for s in c.layers)
    a, b, d, e = (c.layers[i] for i in (0, 1, 2, 7))
    assert (a.mixer, a.heads, a.kv_heads, a.dim, a.vdim, a.decay) == (layered.MIXER_RETENTION, 3, 3, 10, 7, (0.5, 0.9, 0.99))
    assert (a.rot_base, a.rot_dims, a.rot_pairs) == (5000.0, 6, False)
    assert (a.mlp, a.ff, a.act, a.act_limit, a.act_alpha) == (layered.MLP_GATED, 30, layered.ACT_CLAMPED, 0.8, 1.702)
    assert (b.mixer, b.heads, b.kv_heads, b.dim, b.vdim) == (layered.MIXER_PARALLEL, 6, 3, 12, 9)
    assert (b.scale, b.softcap, b.window, b.sink, b.conv_taps, b.rot_base, b.rot_dims) == (0.3, 17.0, 37, True, 4, 700.0, 8)
    assert (b.r_heads, b.r_dim, b.r_vdim, b.decay_rank, b.left_scale, b.right_scale) == (2, 11, 11, 5, 0.6, 1.4)
    assert (b.mlp, b.ff, b.act, b.experts, b.top, b.group_count, b.group_keep) == (layered.MLP_MOE, 20, layered.ACT_SILU, 12, 2, 4, 2)
    assert (b.shared_ff, b.shared_gate, b.router_correction, b.router_renorm, b.router_softmax) == (26, True, True, True, False)
    assert d.mlp == layered.MLP_NONE and (e.heads, e.rot_dims, e.shared_ff) == (1, 4, 5)
    names = {c.tensor_name(int(n[1:].split('.', 1)[0]), n.split('.', 1)[1]) if n[0] == 'l' else n: s for n, s in c.tensor_shapes().items()}
    assert names == {k: tuple(np.shape(v)) for k, v in w.items()}
    native, keep = c.native('float32')
    assert (native.n_layers, native.loop_add, native.tied_head, native.loop_times) == (8, 1, 1, 0)
    n1 = native.layers[1]
    assert (n1.both_norms, n1.group_count, n1.group_keep, n1.router_correction, n1.router_renorm, n1.shared_gate) == (1, 4, 2, 1, 1, 1)
    assert abs(n1.left_scale - 0.6) < 1e-6 and abs(n1.right_scale - 1.4) < 1e-6
    assert abs(native.layers[0].act_limit - 0.8) < 1e-6 and abs(native.layers[0].decay[2] - 0.99) < 1e-6


def test_reader_without_loop_and_refusals():
    c = layered.FAMILIES['Roravik'](ro.make_config(16, 11, [ro.retention_layer(1, 4, 4, [0.9]), ro.parallel_layer(2, 1, 4, 4, 8, 1, 4)]))
    assert not c.loop_add and [s.loop_pass for s in c.layers] == [-1, -1] and [s.weights_of for s in c.layers] == [-1, -1]
    once = layered.FAMILIES['Roravik'](ro.make_config(16, 11, [ro.retention_layer(1, 4, 4, [0.9])], loop=(0, 1, 1)))
    assert not once.loop_add and len(once.layers) == 1
    for change in (lambda c: c['layers'][0]['mixer'].update(decay=[0.5]), lambda c: c['layers'][0]['mixer']['rot'].update(dims=12),
                   lambda c: c['layers'][1]['mlp']['router']['groups'].update(count=5), lambda c: c['layers'][1]['mlp']['router'].update(top=7),
                   lambda c: c['loop'].update(stop=9)):
        c = copy.deepcopy(_cfg())
        change(c)
        with pytest.raises(ValueError):
            layered.FAMILIES['Roravik'](c)
    for change in (lambda c: c['layers'][1].update(type='attention'), lambda c: c['layers'][0]['mlp'].update(kind='glu')):
        c = copy.deepcopy(_cfg())
        change(c)
        with pytest.raises(NotImplementedError):
            layered.FAMILIES['Roravik'](c)


def test_rotation_pairs_halves_and_keeps_relative_positions():
    x = np.array([[1.0, 0.0, 0.0, 1.0, 5.0]])
    y = ro.rotate_half(x, [2], 4, 100.0)
    a, b = 2.0, 2.0 * 0.1                                           # base^(-2/4) = 0.1; channels 0 and 2, 1 and 3
    assert np.allclose(y[0], [math.cos(a), -math.sin(b), math.sin(a), math.cos(b), 5.0])
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((1, 8)), rng.standard_normal((1, 8))
    near = ro.rotate_half(q, [7], 6, 50.0)[0] @ ro.rotate_half(k, [3], 6, 50.0)[0]
    far = ro.rotate_half(q, [107], 6, 50.0)[0] @ ro.rotate_half(k, [103], 6, 50.0)[0]
    assert abs(near - far) < 1e-9


def test_short_convolution_meets_the_current_token_with_its_last_tap():
    u = np.array([[1.0], [10.0], [100.0]])
    assert np.allclose(ro.short_conv(u, np.array([[3.0, 2.0]])), [[2.0], [23.0], [230.0]])
    assert np.allclose(ro.short_conv(u, np.array([[2.0]])), 2.0 * u)


def test_window_and_sink():
    m = ro.window_mask(5, 2)
    assert m.sum() == 9 and m[3].tolist() == [False, False, True, True, False]
    p = ro.sink_softmax(np.array([[0.0, 7.0], [1.0, 2.0]]), np.tri(2, dtype=bool), 0.5)
    e = np.exp([1.0, 2.0, 0.5])
    assert np.allclose(p[1], e[:2] / e.sum()) and np.allclose(p[0], [1.0 / (1.0 + math.exp(0.5)), 0.0])


def test_recurrences_by_hand_and_across_a_cut():
    rng = np.random.default_rng(1)
    q, k, v = rng.standard_normal((6, 3)), rng.standard_normal((6, 3)), rng.standard_normal((6, 2))
    o, S = ro.retention_recurrence(q, k, v, 0.8)
    assert np.allclose(o[4], sum(0.8 ** (4 - j) * (q[4] @ k[j]) * v[j] for j in range(5)))
    o1, S1 = ro.retention_recurrence(q[:2], k[:2], v[:2], 0.8)
    o2, S2 = ro.retention_recurrence(q[2:], k[2:], v[2:], 0.8, S1)
    assert np.allclose(np.concatenate([o1, o2]), o) and np.allclose(S2, S)
    w, u = rng.uniform(0.1, 0.9, (6, 3)), rng.standard_normal(3)
    o, S = ro.bonus_recurrence(q, k, v, w, u)
    past = sum((q[4] * k[j] * np.prod(w[j + 1:4], axis=0)).sum() * v[j] for j in range(4))      # the token's own decay comes behind its output
    assert np.allclose(o[4], past + (q[4] * u * k[4]).sum() * v[4]) and np.allclose(o[0], (q[0] * u * k[0]).sum() * v[0])
    o1, S1 = ro.bonus_recurrence(q[:3], k[:3], v[:3], w[:3], u)
    o2, S2 = ro.bonus_recurrence(q[3:], k[3:], v[3:], w[3:], u, S1)
    assert np.allclose(np.concatenate([o1, o2]), o) and np.allclose(S2, S)


def test_clamped_feed_forward():
    w = {'gate': np.array([[1.0], [-1.0]]), 'up': np.array([[1.0], [1.0]]), 'down': np.eye(2)}
    y = ro.clamped_ff(np.array([[3.0], [-3.0]]), w, '', 2.0)        # the gate is bounded from above only
    f = lambda g, u: g / (1.0 + math.exp(-1.702 * g)) * (u + 1.0)
    assert np.allclose(y, [[f(2.0, 2.0), f(-3.0, 2.0)], [f(-3.0, -2.0), f(2.0, -2.0)]])


def test_router_groups_correction_and_weights():
    r = {'experts': 6, 'top': 2, 'groups': {'count': 3, 'keep': 1}}
    logit = lambda p: math.log(p / (1 - p))
    z = np.array([[logit(p) for p in (0.9, 0.1, 0.6, 0.7, 0.2, 0.3)]])
    assert np.allclose(ro.route(z, np.zeros(6), r)[0], [0, 0, 0.6 / 1.3, 0.7 / 1.3, 0, 0])      # 1.3 beats the group with the best single expert
    c = np.array([0, 0.5, 0, 0, -2.0, -2.0])
    assert np.allclose(ro.route(z, c, r)[0], [0.9, 0.1, 0, 0, 0, 0])                            # the correction orders, the score weighs
    neg = dict(r, groups={'count': 3, 'keep': 2}, top=3)
    assert np.allclose(ro.route(z, np.full(6, -1.0), neg)[0], np.array([0.9, 0, 0.6, 0.7, 0, 0]) / 2.2)     # a dropped group is minus infinity, not zero


def test_loop_order_and_norms_around_zero():
    assert [(i, a) for i, a in ro.layer_runs(_cfg())] == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    y = ro.norm(np.array([[3.0, 4.0]]), np.array([0.0, 1.0]), 0.0)
    assert np.allclose(y, [[3 / math.sqrt(12.5), 8 / math.sqrt(12.5)]])


FAULTS = {
    'sink': lambda c, w: w.update({'l1.mix.left.sink': np.full(6, -1e9)}),
    'bonus': lambda c, w: w.update({'l1.mix.right.u': np.ones((2, 11))}),
    'window one longer': lambda c, w: c['layers'][1]['mixer']['left']['mask'].update(size=38),
    'softcap': lambda c, w: c['layers'][1]['mixer']['left'].update(softcap=1e9),
    'head decay': lambda c, w: c['layers'][0]['mixer']['decay'].reverse(),
    'correction': lambda c, w: w.update({'l1.mlp.correction': np.zeros(12)}),
    'groups': lambda c, w: c['layers'][1]['mlp']['router']['groups'].update(keep=4),
    'limit': lambda c, w: c['layers'][0]['mlp'].update(limit=50.0),
    'token mix': lambda c, w: w.update({'l1.mix.right.mu.k': np.zeros(44)}),
    'passes': lambda c, w: c['loop'].update(times=2),
    'left scale': lambda c, w: c['layers'][1]['mixer'].update(left_scale=0.7),
    'rotated part': lambda c, w: c['layers'][1]['mixer']['left']['rot'].update(dims=6),
    'shared gate': lambda c, w: w.update({'l1.mlp.shared.sg': np.zeros((1, 44))}),
    'eps': lambda c, w: c['norm'].update(eps=1e-2),
    'logit cap': lambda c, w: c.update(logit_softcap=10.0),
}


@pytest.mark.parametrize('fault', list(FAULTS))
def test_a_fault_in_any_mechanism_moves_the_logits(fault):
    """what the GPU tests compare is sensitive: a mistake planted in the float64 model moves its logits far beyond the fp32 tolerance (3e-5)"""
    cfg, bad = _cfg(), copy.deepcopy(_cfg())
    w = ro.random_weights(cfg, 0)
    bw = dict(w)
    FAULTS[fault](bad, bw)
    toks = np.random.default_rng(0).integers(0, 103, 70).tolist()
    ref = ro.forward(cfg, w, toks)
    assert np.abs(ro.forward(bad, bw, toks) - ref).max() > 1e-3 * ref.std()
