"""Engine of the layered mixer models (`models.MixerConfig`): bfloat16 weights, float32 residual and state.

It is a `DecodeEngine` whose layers are lists of mixer ops instead of the attention block: generation, sampling modes,
token lookahead, chunked prefill, lockstep batches and decode plans are the base class's; this class lays out weights,
row buffers, state and cache, and issues the ops.  The op list is made once (`_program`); a step runs it with the
number of rows and the position filled in, from Python or as a registered decode plan.

Maps: 0 float32 workspace (rows, small parameters), 1 and up bfloat16 weights (rows padded to a multiple of 64 with
zeros), 2 operand rows of multi-row products, 3 float32 recurrent state, 14 key-value cache.
`dtype='bfloat16'`: operand rows and cache in bfloat16.  'float32': both in float32 and every product in float32; the
weights are stored in bfloat16 either way, which is exact for a model file that holds them so.

What a sequence keeps is bounded: recurrent state, convolution inputs and one attention chunk or window per layer, so there is
no cache length to choose and no end to a sequence (positions count up to 2^24, where float32 angles stop being exact).
"""
import numpy as np

from .engine import DecodeEngine
from .safetensors_file import TensorDict


def _up_to(n, m):
    return (n + m - 1) // m * m


class SequenceSlots:
    """Which slot of the state and cache a named sequence has, and how many of its tokens the slot holds.  A slot that
    is given back can be handed out again as it is: a sequence's first token reads nothing of it."""

    def __init__(self, n):
        self.pos = [0] * n
        self._free = list(range(n))
        self._of = {}

    def open(self, name):
        if name not in self._of:
            if not self._free:
                raise RuntimeError(f"all {len(self.pos)} sequence slots are in use")
            s = self._of[name] = self._free.pop(0)
            self.pos[s] = 0
        return self._of[name]

    def close(self, name):
        if name in self._of:
            self._free.append(self._of.pop(name))

    def reset(self):
        self.__init__(len(self.pos))


class MixerEngine(DecodeEngine):
    OPND_MAP, STATE_MAP, CACHE_MAP = 2, 3, 14
    WEIGHT_MAPS = [1] + list(range(4, 14))
    LOGIT_ROWS = 16                 # rows of logits a scoring step computes at a time
    MAX_POS = 1 << 24

    def __init__(self, gpu, cfg, tensors, A=None, dtype="bfloat16", prefill_chunk=512, batch=1, map_elem_limit=(1 << 32) - (1 << 24),
                 decode_plan=True, plan_id=0, lookahead=True, sampling_mode=None, **kw):
        if dtype not in ("bfloat16", "float32"):
            raise ValueError(f"dtype '{dtype}': bfloat16 or float32")
        self.dtype = dtype
        self._map_limit = int(map_elem_limit)
        self._kept = 0
        if isinstance(tensors, dict):
            tensors = TensorDict(tensors)
        super().__init__(gpu, cfg, tensors, A=A, kv_cap=self.MAX_POS, fusion_scheduler_mode='level_batched',
                         decode_plan=decode_plan, plan_id=plan_id, prefill_chunk=max(1, int(prefill_chunk)), batch=batch,
                         lookahead=lookahead, sampling_mode=sampling_mode, **kw)

    # ------------------------------------------------------------------ layout
    def _take_tensors(self, tensors):
        return tensors

    def _build_layout(self):
        """Weight matrices -> (map, offset, rows, columns, stride); what shares an input is stacked.  Shapes are checked
        against the configuration, so that a wrong file fails here and by name."""
        c, t = self.cfg, self.tensors
        for name, want in c.tensors().items():
            if name not in t:
                raise ValueError(f"model file lacks tensor {name}")
            have = t.shape(name)
            if len(have) != len(want) or any(w is not None and w != h for w, h in zip(want, have)):
                raise ValueError(f"tensor {name} has shape {have}, expected {want}")
        self._tied, self._lm_name, self._kind = False, 'head', {'head': 'bf16'}
        self._stacks = {}               # stack key (tuple of names) -> (map, offset, n, k, stride)
        self._pack = []                 # (map, offset, blocks, k, stride)
        self._map_size = {}
        where = [0, 0]                  # weight map index, position

        def place(groups):
            total = sum(n * stride for _, _, n, _, stride in groups)
            if where[1] and where[1] + total > self._map_limit:
                where[:] = [where[0] + 1, 0]
            if where[0] >= len(self.WEIGHT_MAPS):
                raise MemoryError("the model's weights exceed the weight maps")
            for key, blocks, n, k, stride in groups:
                mid = self.WEIGHT_MAPS[where[0]]
                self._stacks[key] = (mid, where[1], n, k, stride)
                self._pack.append((mid, where[1], blocks, k, stride))
                where[1] += n * stride
                self._map_size[mid] = where[1]

        def stack(key, blocks):
            """Matrices under each other; a (gate, up) pair alternates in runs of 16 rows."""
            names = [n for b in blocks for n in (b if isinstance(b, tuple) else (b,))]
            k = t.shape(names[0])[1]
            if any(t.shape(n)[1] != k for n in names):
                raise ValueError(f"stacked tensors differ in width: {names}")
            rows = sum(2 * _up_to(t.shape(b[0])[0], 16) if isinstance(b, tuple) else t.shape(b)[0] for b in blocks)
            return (tuple(key), blocks, rows, k, _up_to(k, 64))

        E = c.n_embd
        for name in ['embed'] + (['bigram'] if c.pairs else []):       # rows back to back, as the embedding op reads them
            n = t.shape(name)[0]
            place([((name,), [name], n, E, E)])
            where[1] = self._map_size[self.WEIGHT_MAPS[where[0]]] = _up_to(where[1], 64)
        if c.pairs and self._stacks[('bigram',)][0] != self._stacks[('embed',)][0]:
            raise MemoryError("the embedding tables exceed one weight map")
        place([stack(['head'], ['head'])])
        for i, L in enumerate(c.layers):
            p = f'l{i}.mix.'
            vec = set(L.mixer.vectors())
            ins = [p + n for n in L.mixer.inputs()]
            rest = [p + n for n, s in L.mixer.tensors(E).items() if len(s) == 2 and n not in vec and p + n not in ins]
            groups = [stack(ins, ins)] + [stack([n], [n]) for n in rest]
            if L.ff is not None:
                m = f'l{i}.mlp.'
                named = lambda b: tuple(m + n for n in b) if isinstance(b, tuple) else m + b
                groups += [stack([m + key], [named(b) for b in blocks]) for key, blocks in L.ff.stacks(E).items()]
            place(groups)
        # float32 vectors; an input projection's biases lie one after the other, as the rows they are added to
        self._vec_runs = [['final.norm']]
        for i, L in enumerate(c.layers):
            p = f'l{i}.mix.'
            self._vec_runs += [[n] for n in c.norms(i)] + [[p + n] for n in L.mixer.vectors()]
            self._vec_runs += [[p + n for n in L.mixer.biases()]] if L.mixer.biases() else []
            self._vec_runs += [[f'l{i}.mlp.{n}'] for n in L.ff.vectors()] if L.ff is not None else []
        if self.dtype == "float32":
            bad = [n for g in self._pack for b in g[2] for n in (b if isinstance(b, tuple) else (b,)) if not t.is_bf16_exact(n)]
            if bad:
                raise ValueError(f"dtype float32: tensor {bad[0]} does not fit bfloat16 storage without rounding")
        self._map_of = {'head': self._stacks[('head',)][0]}

    # ------------------------------------------------------------------ workspace
    def _alloc_workspace(self):
        c, M, E = self.cfg, self._chunk, self.cfg.n_embd
        self._ws = {}
        self._fused_groups = 1
        self._c1, self._c_tok1 = {}, None
        pos = 0

        def take(n, align=64):
            nonlocal pos
            pos = _up_to(pos, align)
            pos += n
            return pos - n

        # rows: every buffer holds M rows, as wide as the widest layer needs
        width = {"hidden": E}
        if c.post_norm:
            width.update(hidden2=E, branch=E)
        single, self._operands = {}, {}
        shape = lambda n: self.tensors.shape(n)
        for i, L in enumerate(c.layers):
            p = f'l{i}.mix.'
            w = dict(L.mixer.widths(lambda n: shape(p + n)))
            w["x"] = sum(shape(p + n)[0] for n in L.mixer.inputs())
            if L.ff is not None:
                w.update(L.ff.widths(E))
                for n, v in L.ff.single(E).items():
                    single[n] = max(single.get(n, 0), v)
                for key, v in L.ff.operands().items():
                    self._operands[key] = max(self._operands.get(key, 0), v)
            for n, v in w.items():
                width[n] = max(width.get(n, 0), E if v is None else v)
        self._rows = {}
        for n, w in width.items():
            w = w if n == "hidden" else _up_to(w, 4)      # (the embedding op writes its rows back to back)
            self._rows[n] = (take(M * w), w)
        for n, w in single.items():
            self._rows[n] = (take(w), w)
        self._rows["logit_rows"] = (take(max(self.LOGIT_ROWS, self._batch) * c.n_vocab), c.n_vocab)
        for name, sz in self._sample_slots():
            self._span(name, sz, take(sz))
        self._rows["logits"] = (self._ws['logits'][2], c.n_vocab)
        self._ws['hidden'] = self._ws['normed'] = (0, E, self._rows["hidden"][0])
        self._c_tok_pos = take(M)
        self._c_tok_locs = np.arange(self._c_tok_pos, self._c_tok_pos + M, dtype=np.uint32)
        self._tok_rows_h = self._up(self._c_tok_locs)
        self._hid_locs = np.arange(self._rows["hidden"][0], self._rows["hidden"][0] + E, dtype=np.uint32)
        self._alloc_sample_handles()
        self._vec_off = {}
        for run in self._vec_runs:
            for j, n in enumerate(run):
                self._vec_off[n] = take(int(np.prod(self.tensors.shape(n))), 1 if j else 64)
        self._consts = {}
        self._const_at = take(sum(L.mixer.const_size() for L in c.layers))
        self._ws_total = pos
        # operand rows: one region for what a product normalises or converts, one per kind of activation
        kmax = max(s[4] for k, s in self._stacks.items() if k != ('embed',))
        self._opnd_total = M * kmax
        self._operand_at = {}
        for key, n in self._operands.items():
            self._operand_at[key] = self._opnd_total
            self._opnd_total += M * n
        runs = [c.layers[i].mixer for i in c.runs()]
        self._prev_at = sum(m.state_size() for m in runs)        # (a bigram table's previous token)
        self.state_per_seq = _up_to(self._prev_at + (1 if c.pairs else 0), 64) or 64
        self.cache_per_seq = _up_to(sum(m.cache_size() for m in runs), 64) or 64
        self.slots = SequenceSlots(self._batch)

    # ------------------------------------------------------------------ upload
    def _upload_all(self):
        g, A, t = self.gpu, self.A, self.tensors
        g.set_dtype(A.DTYPE_F32)
        g.map_create(self.WS_MAP, 1, self._ws_total)
        wide = A.DTYPE_F32 if self.dtype == "float32" else A.DTYPE_BF16
        g.map_create_typed(self.OPND_MAP, wide, 1, self._opnd_total)
        g.map_create_typed(self.STATE_MAP, A.DTYPE_F32, 1, self._batch * self.state_per_seq)
        g.map_create_typed(self.CACHE_MAP, wide, 1, self._batch * self.cache_per_seq)
        for mid, n in self._map_size.items():
            g.map_create_typed(mid, A.DTYPE_BF16, 1, n)
        step = 1 << 24

        def put(mid, off, rows):
            flat = np.ascontiguousarray(rows).reshape(-1)
            for b in range(0, flat.size, step):
                g.scatter_contiguous(mid, off + b, flat[b:b + step])

        for mid, off, blocks, k, stride in self._pack:
            for block in blocks:
                if isinstance(block, tuple):             # 16 gate rows, their 16 up rows, and so on
                    ff = t.shape(block[0])[0]
                    n = _up_to(ff, 16)
                    w = np.zeros((n // 16, 2, 16, stride), np.uint16)
                    for j, name in enumerate(block):
                        one = np.zeros((n, stride), np.uint16)
                        one[:ff, :k] = t.bf16(name)
                        w[:, j] = one.reshape(n // 16, 16, stride)
                else:
                    w = t.bf16(block)
                    if stride != k:
                        pad = np.zeros((w.shape[0], stride), np.uint16)
                        pad[:, :k] = w
                        w = pad
                put(mid, off, w)
                off += w.size
        for n, off in self._vec_off.items():
            g.scatter_contiguous(self.WS_MAP, off, np.ascontiguousarray(t.f32(n)).reshape(-1))

    def _alloc_kv_cache(self):
        self.reset()

    def _upload_locs(self):
        c, A = self.cfg, self.A
        self._program = []
        self._state_at = self._cache_at = 0
        self._emit = self._program
        self._residual, self._added = "hidden", None
        into = lambda: (self.at("branch"), A.EPI_STORE) if c.post_norm else (self.at("hidden"), A.EPI_ADD)
        for i in c.runs():
            L, p = c.layers[i], f'l{i}.mix.'
            ins = [p + n for n in L.mixer.inputs()]
            cols, at = {}, 0
            for n in L.mixer.inputs():
                cols[n] = at
                at += self.tensors.shape(p + n)[0]
            bias = [p + n for n in L.mixer.biases()]
            norm = self.model_norm(f'l{i}.norm1', advance=True)
            self.linear(ins, src=self._src, out=self.at("x"), norm=norm, bias=self.vec(bias[0]) if bias else None)
            L.mixer.core(self, p, cols)
            L.mixer.output(self, p, cols, *into())
            if c.post_norm:
                self._added = f'l{i}.norm1b'
            if L.ff is not None:
                norm = self.model_norm(f'l{i}.norm2', advance=True)
                L.ff.issue(self, f'l{i}.mlp.', norm, *into())
                if c.post_norm:
                    self._added = f'l{i}.norm2b'
        self._heads, self._row_lists = {}, {}
        self._score_h = self._head_spec(0, "logit_rows")
        if c.pairs is not None:
            (_, table), (_, pairs) = self._stacks[('embed',)][:2], self._stacks[('bigram',)][:2]
            self._bigram_h = self._up(A.BigramSpec(
                table=table, vocab=c.n_vocab, width=c.n_embd, dst=self._rows["hidden"][0], scale=c.emb_scale, pairs=pairs,
                buckets=c.pairs.buckets, mul_prev=c.pairs.mul_prev, mul_cur=c.pairs.mul_cur, state_map=self.STATE_MAP,
                prev_off=self._prev_at, seq_stride=self.state_per_seq).words())

    # ------------------------------------------------------------------ what mixers issue their ops through
    def at(self, rows, col=0):
        """(offset, stride) of a row buffer, from column `col` on."""
        off, stride = self._rows[rows]
        return off + col, stride

    def vec(self, name):
        return self._vec_off[name]

    def residual(self):
        """Rows of the residual stream the op being issued reads (its norm says what is still to be added to them)."""
        return self._src

    def operand(self, key):
        return self._operand_at[key]

    def stack(self, names):
        """(map, offset, rows, columns, stride) of stacked matrices."""
        return self._stacks[tuple(names)]

    def const(self, values):
        """Workspace offset of float32 constants (kept once per distinct list)."""
        v = np.asarray(values, np.float64).astype(np.float32)
        key = v.tobytes()
        if key not in self._consts:
            self._consts[key] = self._const_at
            if v.size:
                self.gpu.scatter_contiguous(self.WS_MAP, self._const_at, v)
            self._const_at += v.size
        return self._consts[key]

    def take_state(self, n):
        self._state_at += n
        return self._state_at - n

    def take_cache(self, n):
        self._cache_at += n
        return self._cache_at - n

    @staticmethod
    def norm(groups, wt=0, wt_len=0, gate=None, eps=None, wt_add=0.0):
        d = {"groups": groups, "wt": wt, "wt_len": wt_len, "eps": eps, "wt_add": wt_add}
        if gate is not None:
            d.update(gate=gate[0], gate_stride=gate[1], gate_act=gate[2])
        return d

    def model_norm(self, name, advance=False):
        """Norm of the residual stream.  With norms behind the sublayers the last sublayer's output is still in the `branch`
        rows, ahead of its own norm: whoever reads the stream next adds it.  `advance`: and stores the sum, in the other
        of two row buffers (every workgroup of a launch reads the one while one of them writes the other)."""
        d = self.norm(self.cfg.norm_groups, self.vec(name), self.cfg.n_embd, wt_add=self.cfg.norm_add)
        self._src = self.at(self._residual)
        if self._added is not None:
            (branch, bs) = self.at("branch")
            d.update(branch=branch, branch_stride=bs, branch_wt=self.vec(self._added), branched=1)
            if advance:
                self._residual, self._added = "hidden2" if self._residual == "hidden" else "hidden", None
                d.update(branched=2, res_out=self.at(self._residual)[0], res_stride=self.at(self._residual)[1])
        return d

    def linear_spec(self, names, src, out, norm=None, epi=0, opnd=0, ready=0, out_opnd=(0, 0), bias=None, keep=None, tail=None):
        """(weight map, spec handle) of y = W . f(x); bias: offset of a vector added to y, keep: rows f(x) is also stored in,
        tail: (count, rows) of the ordinary rows behind gate and up pairs."""
        mid, off, n, k, stride = self.stack(names)
        f = dict(norm or {"groups": 0})
        f["eps"] = self.cfg.norm_eps if f.get("eps") is None else f["eps"]
        if bias is not None:
            f.update(bias=bias, biased=1)
        if keep is not None:
            f.update(keep=keep[0], keep_stride=keep[1], kept=1)
        if tail is not None:
            f.update(tail=tail[0], tail_out=tail[1][0], tail_stride=tail[1][1])
        spec = self.A.LinearSpec(w=off, n=n, k=k, k_stride=stride, src=src[0], src_stride=src[1], opnd=opnd, ready=ready, out=out[0],
                                 out_stride=out[1], epi=epi, out_opnd=out_opnd[0], out_opnd_stride=out_opnd[1], **f)
        return mid, self._up(spec.words())

    def linear(self, names, src, out, **kw):
        mid, h = self.linear_spec(names, src, out, **kw)
        self._emit.append((self.A.DECODE_OP_LINEAR, mid, h, 0, 0))

    def experts(self, mid, spec, shared):
        self._emit.append((self.A.DECODE_OP_EXPERTS, mid, self._up(spec.words()), shared, 0))

    def window_attention(self, spec):
        self._emit.append((self.A.DECODE_OP_WINDOW_ATTENTION, 0, self._up(spec.words()), 0, 0))

    def state_space(self, spec):
        self._emit.append((self.A.DECODE_OP_STATE_SPACE, 0, self._up(spec.words()), 0, 0))

    def delta_rule(self, spec, decay, gate):
        assert decay[0] == gate[0]
        self._emit.append((self.A.DECODE_OP_DELTA_RULE, decay[0], self._up(spec.words()), decay[1], gate[1]))

    def retention(self, spec):
        self._emit.append((self.A.DECODE_OP_RETENTION, 0, self._up(spec.words()), 0, 0))

    def chunk_attention(self, spec):
        self._emit.append((self.A.DECODE_OP_CHUNK_ATTENTION, 0, self._up(spec.words()), 0, 0))

    def merge(self, a, b, wa, wb, out, scale, epi):
        ao, stride = self.at(a)
        bo, stride_b = self.at(b)
        assert stride == stride_b
        spec = self.A.MergeSpec(a=ao, b=bo, stride=stride, wa=wa, wb=wb, dst=out[0], dst_stride=out[1], dim=self.cfg.n_embd,
                                eps=self.cfg.norm_eps, scale=scale, store=1 if epi == self.A.EPI_STORE else 0)
        self._emit.append((self.A.DECODE_OP_MERGE_NORM, 0, self._up(spec.words()), 0, 0))

    # ------------------------------------------------------------------ running the op list
    def _run_program(self, n_seq, rows, seq0, pos):
        """`rows` tokens of one sequence, or one token of each of n_seq sequences, from the hidden rows to the hidden rows."""
        g, A, ws, n = self.gpu, self.A, self.WS_MAP, n_seq * rows
        for kind, mid, h0, h1, h2 in self._program:
            if kind == A.DECODE_OP_LINEAR:
                g.linear_dev(ws, self.OPND_MAP, mid, h0, 0, n)
            elif kind == A.DECODE_OP_MERGE_NORM:
                g.merge_norm_dev(ws, h0, n)
            elif kind == A.DECODE_OP_DELTA_RULE:
                g.delta_rule_dev(ws, self.OPND_MAP, mid, h0, h1, h2, n_seq, rows, seq0, pos)
            elif kind == A.DECODE_OP_RETENTION:
                g.retention_dev(ws, h0, n_seq, rows, seq0, pos)
            elif kind == A.DECODE_OP_CHUNK_ATTENTION:
                g.chunk_attention_dev(ws, h0, n_seq, rows, seq0, pos)
            elif kind == A.DECODE_OP_WINDOW_ATTENTION:
                g.window_attention_dev(ws, h0, n_seq, rows, seq0, pos)
            elif kind == A.DECODE_OP_STATE_SPACE:
                g.state_space_dev(ws, h0, n_seq, rows, seq0, pos)
            else:
                g.experts_dev(ws, self.OPND_MAP, mid, h0, h1, n)

    def _ops_for(self, n_seq):
        A, P = self.A, self.A.DECODE_RUNTIME_POS
        ops = []
        for kind, mid, h0, h1, h2 in self._program:
            op = A.DecodePlanOp(kind=kind, map_id=self.WS_MAP, map_id2=mid, op_code=self.OPND_MAP, h0=h0, h1=h1, h2=h2, u0=n_seq)
            if kind not in (A.DECODE_OP_LINEAR, A.DECODE_OP_MERGE_NORM, A.DECODE_OP_EXPERTS):
                op.u1, op.u2, op.u3 = 1, 0, P
            ops.append(op)
        return ops

    def _plan_ops(self):
        return self._ops_for(1)

    def _lockstep_plan_ops(self, m):
        return self._ops_for(m)

    # ------------------------------------------------------------------ steps
    def _head_spec(self, row, out):
        norm = self.model_norm('final.norm')
        src, stride = self._src
        if row and norm.get("branched"):
            norm["branch"] += row * norm["branch_stride"]
        return self.linear_spec(['head'], src=(src + row * stride, stride), out=self.at(out), norm=norm)

    def _head(self, row):
        """Spec handle of final norm and LM head over hidden row `row`, logits to the `logits` slot."""
        if row not in self._heads:
            self._heads[row] = self._head_spec(row, "logits")
        return self._heads[row]

    def _follows(self, slot, pos, n):
        if self.slots.pos[slot] != pos:
            raise RuntimeError(f"sequence slot {slot} holds {self.slots.pos[slot]} tokens; a step at position {pos} cannot follow")
        if pos + n > self.MAX_POS:
            raise RuntimeError(f"sequence of {pos + n} tokens: at most {self.MAX_POS}")

    def _advance(self, slot, pos, n):
        self._follows(slot, pos, n)
        self.slots.pos[slot] = pos + n

    def _token_feed(self):
        if self._feed is None:
            mid, off = self._stacks[('embed',)][:2]
            self._feed = {'src': (mid, off), 'tok_h': self._up(self._sample_locs), 'tok_hs': {self._batch: self._tok_rows_h}}
        return self._feed

    def _check_tokens(self, toks):
        toks = np.asarray(toks, np.int64)
        if toks.size and (toks.min() < 0 or toks.max() >= self.cfg.n_vocab):
            raise ValueError(f"token ids must lie in 0 .. {self.cfg.n_vocab - 1}")
        return toks.astype(np.float32)

    def _embed(self, toks, n_seq, rows, seq0, pos):
        """Residual rows of `rows` tokens of one sequence, or of one token of each of n_seq sequences."""
        self.gpu.scatter_contiguous(self.WS_MAP, self._c_tok_pos, self._check_tokens(toks))
        self._embed_rows(self._tok_rows_h, n_seq, rows, seq0, pos, False)

    def _embed_rows(self, tok_h, n_seq, rows, seq0, pos, post):
        """The same for tokens that are in their slots; `post`: the launch also hands them to the host."""
        c, g, (mid, off) = self.cfg, self.gpu, self._token_feed()['src']
        if c.pairs is not None:
            t = g.embed_bigram_dev(self.WS_MAP, mid, self._bigram_h, tok_h, n_seq, rows, seq0, pos, post)
        else:
            t = (g.embed_post_tokens_dev if post else g.embed_tokens_dev)(self.WS_MAP, mid, tok_h, off, self._rows["hidden"][0], n_seq * rows,
                                                                           c.n_embd, c.n_vocab, float(c.emb_scale))
        if post:
            self._feed_ticket = t

    def _stage_token(self, tok, from_device):
        self._next = None if from_device else tok

    def _issue_embedding(self, from_device, pos):
        self._follows(0, pos, 1)
        if from_device:
            self._embed_rows(self._token_feed()['tok_h'], 1, 1, 0, pos, True)
        else:
            self._embed([self._next], 1, 1, 0, pos)

    def _issue_layers(self, pos):
        self._advance(0, pos, 1)
        if self._plan_id is not None:
            self.gpu.decode_step(self._plan_id, pos, pos + 1)
        else:
            self._run_program(1, 1, 0, pos)

    def _issue_argmax(self, normed_h):
        mid, h = self._head(0)
        self.gpu.linear_argmax_dev(self.WS_MAP, self.OPND_MAP, mid, h, self._feed['tok_h'], 1)

    def _issue_logits(self, normed_h):
        mid, h = self._head(0)
        self.gpu.linear_dev(self.WS_MAP, self.OPND_MAP, mid, h, 0, 1)

    def _head_argmax_built(self):
        return hasattr(self.gpu, 'linear_argmax_dev')

    def _forward_chunk(self, toks, pos0, sample=True, seq=0, lockstep=False, from_device=False):
        """m prompt tokens of sequence `seq` at positions pos0 .. in one pass, or (`lockstep`) one token of each of the
        first m sequences, all at position pos0; see the base class."""
        g, ws = self.gpu, self.WS_MAP
        m = self._batch if from_device else len(toks)
        if m == 0 or m > self._chunk:
            raise RuntimeError(f"chunk of {m} tokens does not fit prefill_chunk={self._chunk}")
        g.batch_begin()
        for s in range(m if lockstep else 1):
            self._advance(s if lockstep else seq, pos0, 1 if lockstep else m)
        n_seq, rows, seq0 = (m, 1, 0) if lockstep else (1, m, seq)
        if from_device:
            self._embed_rows(self._token_feed()['tok_hs'][m], n_seq, rows, seq0, pos0, True)
        else:
            self._embed(toks, n_seq, rows, seq0, pos0)
        if lockstep and self._ls_plan_id is not None and m == self._batch:
            g.decode_step(self._ls_plan_id, pos0, pos0 + 1)
        elif lockstep:
            self._run_program(m, 1, 0, pos0)
        else:
            self._run_program(1, m, seq, pos0)
        if lockstep:
            mid, h = self._score_h
            g.linear_argmax_dev(ws, self.OPND_MAP, mid, h, self._tok_rows_h, m)
        elif sample:
            mid, h = self._head(m - 1)
            g.linear_argmax_dev(ws, self.OPND_MAP, mid, h, self._feed['tok_h'], 1)
            self._sample_token_ready = True
        g.batch_end()

    def reset(self):
        keep, self._kept = self._kept, 0
        self.slots.reset()
        self.slots.pos[0] = keep
        self._sample_token_ready = False

    def _usable_prefix(self, n, n_prompt):
        """A recurrent state cannot be wound back: a prefix is kept only if the slot holds exactly its tokens."""
        self._kept = n if 0 < n < n_prompt and self.slots.pos[0] == n else 0
        return self._kept

    # ------------------------------------------------------------------ scoring
    def score(self, name, tokens, want=()):
        """Feed a named sequence its next tokens; the logits [len(want), n_vocab] at the places `want` among them.  The
        sequence gets a slot with its first tokens and keeps it until `release`."""
        slot = self.slots.open(name)
        tokens = [int(t) for t in tokens]
        self._check_tokens(tokens)
        out = np.empty((len(want), self.cfg.n_vocab), np.float32)
        for lo in range(0, len(tokens), self._chunk):
            part = tokens[lo:lo + self._chunk]
            if len(part) == 1 and slot == 0:
                self._forward(part[0], self.slots.pos[slot], sample=False)
            else:
                self._forward_chunk(part, self.slots.pos[slot], sample=False, seq=slot)
            here = [(i, w - lo) for i, w in enumerate(want) if lo <= w < lo + len(part)]
            for b in range(0, len(here), self.LOGIT_ROWS):
                idx = here[b:b + self.LOGIT_ROWS]
                out[[i for i, _ in idx]] = self._logits_of_rows([r for _, r in idx])
        return out

    def release(self, name):
        self.slots.close(name)

    def _logits_of_rows(self, rows):
        g, n = self.gpu, len(rows)
        r = np.asarray(rows, np.uint32)
        if n in self._row_lists:
            g.upload_dev(r, handle=self._row_lists[n])
        else:
            self._row_lists[n] = self._up(r)
        mid, h = self._score_h
        g.linear_dev(self.WS_MAP, self.OPND_MAP, mid, h, self._row_lists[n], n)
        off = self._rows["logit_rows"][0]
        return g.gather(self.WS_MAP, np.arange(off, off + n * self.cfg.n_vocab, dtype=np.uint32)).view(np.float32).reshape(n, -1)

    def read_rows(self, name, n, width=None):
        """The first n rows of a row buffer (tests, debugging)."""
        off, stride = self._rows[name]
        r = self.gpu.gather(self.WS_MAP, np.arange(off, off + n * stride, dtype=np.uint32)).view(np.float32).reshape(n, stride)
        return r[:, :width or stride].copy()
