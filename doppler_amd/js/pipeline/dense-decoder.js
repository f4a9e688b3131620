// Decoder with dense bf16 weights: the JavaScript side of doppler_amd/dense_decoder.py.  Layers are sequential (sublayers.js) or parallel:
//   x <- x + mixer(norm(x)) + ff(norm(x))
// is two products: [q | k | v | gate | up] = W_in norm(x), and x += W_out [attention | act(up)].  Head sizes are padded
// to multiples of 8 and every k extent to a multiple of 64 with zeros.
import {
  createTensor, acquireBuffer, releaseBuffer, recordEmbedSum, recordRMSNormRows, recordDenseMatmul, recordDenseGemv,
  recordDenseLmHeadArgmax, packAttnSpec, recordAttnSpecKVWrite, recordAttnSpecPrefill, recordAttnSpecDecode, recordCheckFiniteness,
} from '../kernel-selector.js';
import { getNative } from '../native.js';
import { SequentialLayer } from './sublayers.js';
import { TextDecoder, bufferWindow, upload } from './text-decoder.js';

const GEMV_MAX_K = 32768;
const up = (n, m) => Math.ceil(n / m) * m;

// src rows [heads * size] of `cols` elements into dst (row stride ld) from row `at` on, heads `padded` rows apart
function placeHeads(dst, ld, at, src, heads, size, padded, cols) {
  for (let h = 0; h < heads; h++) {
    for (let r = 0; r < size; r++) {
      dst.set(src.subarray((h * size + r) * cols, (h * size + r + 1) * cols), (at + h * padded + r) * ld);
    }
  }
}

function stackLayer(mixer, mlp, w, hidden) {
  const H = mixer.heads, G = mixer.kvHeads, d = mixer.dim, e = mixer.vdim;
  const D = up(d, 8), VD = up(e, 8), ff = mlp ? mlp.ff : 0;
  const g = {
    D, VD, ff, kOffset: H * D, vOffset: (H + G) * D, gateOffset: mixer.gate ? (H + G) * D + G * VD : -1,
    nFirst: (H + G) * D + G * VD + (mixer.gate ? up(H, 8) : 0), kx: up(hidden, 64), k2: up(H * VD + ff, 64), attnCols: H * VD,
  };
  g.n = g.nFirst + ff;
  const wIn = new Uint16Array(g.n * g.kx), bias = new Float32Array(g.nFirst), wOut = new Uint16Array(hidden * g.k2);
  for (const [name, heads, size, padded, at] of [['q', H, d, D, 0], ['k', G, d, D, g.kOffset], ['v', G, e, VD, g.vOffset]]) {
    placeHeads(wIn, g.kx, at, w[name], heads, size, padded, hidden);
    if (w[name + 'Bias']) placeHeads(bias, 1, at, w[name + 'Bias'], heads, size, padded, 1);
  }
  if (mixer.gate) placeHeads(wIn, g.kx, g.gateOffset, w.gate, 1, H, H, hidden);
  if (mlp) placeHeads(wIn, g.kx, g.nFirst, w.up, 1, ff, ff, hidden);
  for (let n = 0; n < hidden; n++) {
    for (let h = 0; h < H; h++) wOut.set(w.o.subarray((n * H + h) * e, (n * H + h + 1) * e), n * g.k2 + h * VD);
    if (mlp) wOut.set(w.down.subarray(n * ff, (n + 1) * ff), n * g.k2 + g.attnCols);
  }
  return { g, wIn, bias, wOut };
}

export class DenseTextDecoder extends TextDecoder {
  // config: {hidden, vocab, eps, logitScale, maxPositions, maxSeq, compute: 'bf16'|'f32', bigram: {buckets, mulPrev, mulCur}|null,
  //          layers: [{mixer: {heads, kvHeads, dim, vdim, window, scale, logBias, valueNorm, gate}, mlp: {ff, activation}|null}, or
  //                   {sequential: true, mixer: {type, ..}, mlp: {type, ..}|null}]}
  // weights: {embed, bigram, pos, head (Uint16Array bf16 bits), finalNorm, layers: [{norm, qBias, kBias, vBias, biasR1, biasR2
  //           (Float32Array), q, k, v, gate, o, up, down (Uint16Array)}, or what SequentialLayer takes]}
  constructor(config, weights) {
    super(config);
    const c = config;
    if (c.maxPositions && c.maxSeq > c.maxPositions) throw new Error(`[DenseTextDecoder] maxSeq=${c.maxSeq} exceeds the model's ${c.maxPositions} positions`);
    this.operand = c.compute === 'f32' ? 'f32' : 'bf16';
    const cacheDtype = this.operand === 'bf16' ? 'f16' : 'f32', cacheBytes = this.operand === 'bf16' ? 2 : 4;
    this.kx = up(c.hidden, 64);
    if (this.kx > GEMV_MAX_K) throw new Error(`[DenseTextDecoder] widths beyond ${GEMV_MAX_K} are not served by this host`);
    const padded = (v) => { const out = new Float32Array(this.kx); out.set(v); return upload(out, 'norm'); };
    let workspace = 256, qkv = 1;
    this.mixed = new Map();
    this.scratchBuffers = new Map();
    this.rotaryTables = new Map();
    this.operandBytes = this.operand === 'bf16' ? 2 : 4;
    const earlier = [];
    const keep = (layer) => { earlier.push(layer); return layer; };
    this.layers = weights.layers.map((w, i) => {
      if (c.layers[i].sequential) return keep({ sublayers: new SequentialLayer(this, c.layers[i], w, earlier.map((l) => l.sublayers)) });
      const m = c.layers[i].mixer, mlp = c.layers[i].mlp;
      const { g, wIn, bias, wOut } = stackLayer(m, mlp, w, c.hidden);
      if (g.k2 > GEMV_MAX_K) throw new Error(`[DenseTextDecoder] layer ${i}: rows of ${g.k2} are not served by this host`);
      const l = {
        wIn: upload(wIn, `L${i}.in`), bias: upload(bias, `L${i}.bias`), wOut: upload(wOut, `L${i}.out`), norm: padded(w.norm),
        cacheK: acquireBuffer(c.maxSeq * m.kvHeads * g.D * cacheBytes, undefined, 'kv_k'),
        cacheV: acquireBuffer(c.maxSeq * m.kvHeads * g.VD * cacheBytes, undefined, 'kv_v'),
      };
      if (m.logBias) { l.r1 = upload(w.biasR1, 'bias_r1'); l.r2 = upload(w.biasR2, 'bias_r2'); }
      const spec = packAttnSpec({
        heads: m.heads, kvHeads: m.kvHeads, D: g.D, VD: g.VD, valueDim: m.vdim, window: m.window, cacheDtype, valueNorm: m.valueNorm,
        kOffset: g.kOffset, vOffset: g.vOffset, gateOffset: g.gateOffset, ldQkv: g.nFirst, scale: m.scale, valueEps: c.eps,
        biasR1: l.r1, biasR2: l.r2,
      });
      workspace = Math.max(workspace, getNative().attnSpecWorkspaceBytes(m.heads, g.VD, c.maxSeq));
      qkv = Math.max(qkv, g.nFirst);
      const key = `${g.attnCols + g.ff}/${g.k2}`;
      if (!this.mixed.has(key)) this.mixed.set(key, this.zeroed(g.k2 * 4, 'mixed'));
      return keep({ buffers: l, g, spec, key, activation: mlp ? mlp.activation : 'none' });
    });
    this.tables = {
      embed: upload(weights.embed, 'embed'), bigram: c.bigram ? upload(weights.bigram, 'bigram') : null,
      pos: c.maxPositions ? upload(weights.pos, 'pos') : null, finalNorm: padded(weights.finalNorm),
    };
    const head = new Uint16Array(c.vocab * this.kx);
    placeHeads(head, this.kx, 0, weights.head, 1, c.vocab, c.vocab, c.hidden);
    this.tables.head = upload(head, 'head');
    this.step = { x: this.zeroed(this.kx * 4, 'residual'), qkv: this.zeroed(qkv * 4, 'qkv'), attn: this.zeroed(workspace, 'attn_ws') };
    this.qkvN = qkv;
    this.batch = null;
  }

  // the padding behind a buffer's rows must be zero, also in memory the pool hands out again
  zeroed(bytes, label) {
    const b = acquireBuffer(up(bytes, 4), undefined, label);
    getNative().fillZero(b.ptr, 0, up(bytes, 4));
    return b;
  }

  // A buffer all layers share, by name and row width (what lies behind a row's elements stays zero), grown to the most rows asked for.
  scratch(name, width, count, elementBytes) {
    const key = `${name}/${width}/${elementBytes}`, bytes = width * count * elementBytes;
    const held = this.scratchBuffers.get(key);
    if (held && held.size >= bytes) return held;
    if (held) releaseBuffer(held);
    const buffer = this.zeroed(bytes, name);
    this.scratchBuffers.set(key, buffer);
    return buffer;
  }

  rotary(base, dims, make) {
    const key = `${base}/${dims}`;
    if (!this.rotaryTables.has(key)) {
      const t = make(base, dims, this.config.maxSeq);
      this.rotaryTables.set(key, { cos: upload(t.cos, 'cos'), sin: upload(t.sin, 'sin') });
    }
    return this.rotaryTables.get(key);
  }

  carriesState() {
    return this.layers.some((l) => l.sublayers && l.sublayers.recurrent);
  }

  deviceKvLenServed() {
    return true;
  }

  embedding(ids, indexOffset, prev, output, numTokens, startPos, kvLenBuffer) {
    const c = this.config, t = this.tables;
    return {
      ids, indexOffset, prev, embed: t.embed, vocab: c.vocab, bigram: t.bigram ? Object.assign({ table: t.bigram }, c.bigram) : null,
      pos: t.pos ? { table: t.pos, count: c.maxPositions } : null, output, ldOut: this.kx, numTokens, hidden: c.hidden, startPos, kvLenBuffer,
    };
  }

  async recordEmbedding(recorder, temps, ids, prev, pos, options) {
    recordEmbedSum(recorder, this.embedding(ids, 0, prev, this.step.x, 1, pos, options.deviceKvLen ? bufferWindow(this.ids, 4, 4) : null));
    return createTensor(this.step.x, 'f32', [1, this.kx], 'residual');
  }

  async recordLayers(recorder, temps, x, pos, options) {
    const c = this.config, s = this.step;
    const kvLen = options.deviceKvLen ? bufferWindow(this.ids, 4, 4) : null;
    for (let li = 0; li < this.layers.length; li++) {
      const layer = this.layers[li];
      if (layer.sublayers) layer.sublayers.step(recorder, pos, kvLen);
      else this.recordParallelLayer(recorder, layer, pos, kvLen);
      if (this.finitenessGuard) {
        recordCheckFiniteness(recorder, x, c.hidden, this.finitenessStatus, li, pos, this.finitenessAbsThreshold);
      }
    }
    return x;
  }

  recordParallelLayer(recorder, { buffers: l, g, spec, key, activation }, pos, kvLen) {
    const c = this.config, s = this.step, mixed = this.mixed.get(key);
    recordDenseGemv(recorder, {
      input: s.x, normWeight: l.norm, hidden: c.hidden, eps: c.eps, weight: l.wIn, ldw: g.kx, N: g.n, K: g.kx, bias: l.bias, output: s.qkv,
      nFirst: g.nFirst, output2: g.ff ? bufferWindow(mixed, 4 * g.attnCols, 4 * g.ff) : null, activation,
    });
    recordAttnSpecDecode(recorder, spec, s.qkv, l.cacheK, l.cacheV, mixed, pos, kvLen, c.maxSeq, s.attn);
    recordDenseGemv(recorder, { input: mixed, weight: l.wOut, ldw: g.k2, N: c.hidden, K: g.k2, residual: s.x, output: s.x, nFirst: c.hidden });
  }

  async recordNormedLmHead(recorder, temps, row, tokenOut, tokenIndex, logitsOutput) {
    const c = this.config, t = this.tables;
    recordDenseLmHeadArgmax(recorder, {
      input: row, normWeight: t.finalNorm, hidden: c.hidden, eps: c.eps, weight: t.head, ldw: this.kx, vocab: c.vocab, K: this.kx,
      alpha: c.logitScale, outputBuffer: tokenOut, outputIndex: tokenIndex, logitsOutput,
    });
  }

  async recordPrefillChunk(recorder, temps, ids, part, pos) {
    const c = this.config, T = part.length, elem = this.operand === 'bf16' ? 2 : 4;
    if (!this.batch || this.batch.rows < T) {
      this.releaseBatch();
      const mixed = new Map();
      for (const { g, key } of this.layers.filter((l) => !l.sublayers)) {
        if (!mixed.has(key)) mixed.set(key, this.zeroed(T * g.k2 * elem, 'prefill_mixed'));
      }
      this.batch = {
        rows: T, mixed, x: this.zeroed(T * this.kx * 4, 'prefill_x'), normed: this.zeroed(T * this.kx * elem, 'prefill_normed'),
        qkv: this.zeroed(T * this.qkvN * 4, 'prefill_qkv'),
      };
    }
    const b = this.batch;
    recordEmbedSum(recorder, this.embedding(ids, 1, ids, b.x, T, pos, null));
    for (const layer of this.layers) {
      if (layer.sublayers) {
        layer.sublayers.rows(recorder, b.x, T, pos);
        continue;
      }
      const { buffers: l, g, spec, key, activation } = layer;
      const mixed = b.mixed.get(key);
      recordRMSNormRows(recorder, {
        input: b.x, ldIn: this.kx, rows: null, weight: l.norm, output: b.normed, dtype: this.operand, ldOut: this.kx, count: T,
        hidden: c.hidden, eps: c.eps,
      });
      recordDenseMatmul(recorder, {
        input: b.normed, dtype: this.operand, lda: this.kx, weight: l.wIn, ldw: g.kx, M: T, N: g.n, K: g.kx, bias: l.bias, output: b.qkv,
        ldc: g.nFirst, nFirst: g.nFirst, output2: g.ff ? bufferWindow(mixed, elem * g.attnCols, mixed.size - elem * g.attnCols) : null,
        dtype2: this.operand, ldc2: g.k2, activation,
      });
      recordAttnSpecKVWrite(recorder, spec, b.qkv, l.cacheK, l.cacheV, T, pos);
      recordAttnSpecPrefill(recorder, spec, b.qkv, l.cacheK, l.cacheV, mixed, this.operand, g.k2, T, pos);
      recordDenseMatmul(recorder, {
        input: mixed, dtype: this.operand, lda: g.k2, weight: l.wOut, ldw: g.k2, M: T, N: c.hidden, K: g.k2, residual: b.x, output: b.x,
        ldc: this.kx, nFirst: c.hidden,
      });
    }
    return { buffer: b.x, rowFloats: this.kx };
  }

  releaseBatch() {
    if (!this.batch) return;
    for (const b of [this.batch.x, this.batch.normed, this.batch.qkv].concat(Array.from(this.batch.mixed.values()))) releaseBuffer(b);
    this.batch = null;
  }

  releaseWeights() {
    this.releaseBatch();
    for (const l of this.layers) (l.sublayers ? l.sublayers.ownBuffers() : Object.values(l.buffers)).forEach(releaseBuffer);
    const shared = [].concat(...Array.from(this.rotaryTables.values()).map((t) => [t.cos, t.sin]), Array.from(this.scratchBuffers.values()));
    for (const b of Array.from(this.mixed.values()).concat(Object.values(this.step), Object.values(this.tables), shared)) releaseBuffer(b);
  }
}
