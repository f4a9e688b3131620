// Layers whose sublayers run one after the other: the JavaScript side of doppler_amd/sublayers.py, with the same stacking,
// padding and launches.
//   x <- x + ls1 * mixer(norm1(x));   x <- x + ls2 * ff(norm2(x))
// A sublayer has step(recorder, pos, kvLen) for one token and rows(recorder, x, count, pos) for a portion; `buffers` are its own.
import {
  recordRMSNormRows, packLatent, packMlstm, packExperts, recordDenseMatmulScaled, recordDenseGemvScaled, recordDenseGemvHeads,
  recordHeadNormGate, recordLatentRows, recordLatentPrefill, recordLatentDecode, recordMlstmStep, recordMlstmPrefill, recordExpertsStep,
  recordExpertsPrefill,
} from '../kernel-selector.js';
import { getNative, DTYPE } from '../native.js';
import { bufferWindow, upload } from './text-decoder.js';

const GEMV_MAX_K = 32768, GEMV_MAX_HEADS = 256;
const up = (n, m) => Math.ceil(n / m) * m;

// src rows [heads][size] of `cols` elements into dst (row stride ld) from row `at` on, heads `padded` rows apart; `from` of `of` rows
// of a source head are skipped
function placeRows(dst, ld, at, src, heads, size, padded, cols, from = 0, of = size) {
  for (let h = 0; h < heads; h++) {
    for (let r = 0; r < size; r++) {
      const s = (h * of + from + r) * cols;
      dst.set(src.subarray(s, s + cols), (at + h * padded + r) * ld);
    }
  }
}

// output projection [hidden][heads * size] -> [hidden][k], heads `padded` columns apart
function padOut(o, hidden, heads, size, padded, k) {
  const out = new Uint16Array(hidden * k);
  for (let n = 0; n < hidden; n++) {
    for (let h = 0; h < heads; h++) out.set(o.subarray((n * heads + h) * size, (n * heads + h + 1) * size), n * k + h * padded);
  }
  return out;
}

// bf16 bits to the nearest f16 bits (ties to even)
export function bf16ToF16(bits) {
  const out = new Uint16Array(bits.length);
  for (let i = 0; i < bits.length; i++) {
    const b = bits[i], sign = b & 0x8000, e = ((b >> 7) & 0xFF) - 112, m = b & 0x7F;
    if (((b >> 7) & 0xFF) === 0xFF) out[i] = sign | 0x7C00 | (m ? 0x200 : 0);
    else if (e >= 31) out[i] = sign | 0x7C00;
    else if (e > 0) out[i] = sign | (e << 10) | (m << 3);
    else if (e < -10) out[i] = sign;
    else {
      const full = (0x80 | m) << 3, shift = 1 - e, low = full & ((1 << shift) - 1), half = 1 << (shift - 1);
      let q = full >> shift;
      if (low > half || (low === half && (q & 1))) q++;
      out[i] = sign | q;
    }
  }
  return out;
}

// cos and sin [positions][dims / 2] of the angles p base^(-2 i / dims)
function rotaryTables(base, dims, positions) {
  const half = dims / 2, cos = new Float32Array(positions * half), sin = new Float32Array(positions * half);
  for (let p = 0; p < positions; p++) {
    for (let i = 0; i < half; i++) {
      const a = p * Math.pow(base, (-2 * i) / dims);
      cos[p * half + i] = Math.cos(a);
      sin[p * half + i] = Math.sin(a);
    }
  }
  return { cos, sin };
}

class Sublayer {
  // dec: the decoder; norm: the sublayer's norm weights; ls: its layer scale
  constructor(dec, norm, ls) {
    this.dec = dec;
    this.hidden = dec.config.hidden;
    this.kx = dec.kx;
    this.eps = dec.config.eps;
    const padded = new Float32Array(this.kx);
    padded.set(norm);
    this.buffers = { norm: upload(padded, 'norm'), ls: upload(ls, 'layer_scale') };
  }

  checkRow(k) {
    if (k > GEMV_MAX_K) throw new Error(`[sublayer] rows of ${k} elements are longer than the ${GEMV_MAX_K} a decode step holds`);
  }

  normedGemv(recorder, weight, n, options) {
    recordDenseGemvScaled(recorder, Object.assign({
      input: this.dec.step.x, normWeight: this.buffers.norm, hidden: this.hidden, eps: this.eps, weight, ldw: this.kx, N: n, K: this.kx,
    }, options));
  }

  outGemv(recorder, input, weight, k) {
    const x = this.dec.step.x;
    recordDenseGemvScaled(recorder, {
      input, weight, ldw: k, N: this.hidden, K: k, columnScale: this.buffers.ls, residual: x, output: x, nFirst: this.hidden,
    });
  }

  normedRows(recorder, x, count) {
    const d = this.dec, out = d.scratch('normed', this.kx, count, d.operandBytes);
    recordRMSNormRows(recorder, {
      input: x, ldIn: this.kx, rows: null, weight: this.buffers.norm, output: out, dtype: d.operand, ldOut: this.kx, count, hidden: this.hidden, eps: this.eps,
    });
    return out;
  }

  inRows(recorder, input, count, weight, n, options) {
    recordDenseMatmulScaled(recorder, Object.assign({ input, dtype: this.dec.operand, lda: this.kx, weight, ldw: this.kx, M: count, N: n, K: this.kx }, options));
  }

  outRows(recorder, input, k, weight, x, count) {
    recordDenseMatmulScaled(recorder, {
      input, dtype: this.dec.operand, lda: k, weight, ldw: k, M: count, N: this.hidden, K: k, columnScale: this.buffers.ls, residual: x, output: x,
      ldc: this.kx, nFirst: this.hidden,
    });
  }
}

class LatentAttention extends Sublayer {
  constructor(dec, m, w, norm, ls, lender) {
    super(dec, norm, ls);
    const H = m.heads, d = m.dim, rot = m.rotDim, e = m.vdim, rank = m.kvRank;
    const D = up(d, 8), R = up(rot, 32), VD = up(e, 8), C = up(rank, 64), half = dec.operand === 'bf16', b = this.buffers;
    const qRows = H * (D + R);
    this.nIn = qRows + (lender ? 0 : C + R);
    this.ld = up(Math.max(this.nIn, H * VD), 8);
    this.k2 = up(H * VD, 64);
    this.checkRow(Math.max(this.kx, this.k2));
    const wIn = new Uint16Array(this.nIn * this.kx);
    placeRows(wIn, this.kx, 0, w.q, H, d, D + R, this.hidden, 0, d + rot);
    placeRows(wIn, this.kx, D, w.q, H, rot, D + R, this.hidden, d, d + rot);
    if (!lender) {
      placeRows(wIn, this.kx, qRows, w.dkv, 1, rank, rank, this.hidden);
      placeRows(wIn, this.kx, qRows + C, w.dkv, 1, rot, rot, this.hidden, rank);
      b.latentNorm = upload(w.latentNorm, 'latent_norm');
      // the products read whole k tiles: what they touch behind the last row is zero too
      b.cache = dec.zeroed((dec.config.maxSeq + 1) * (C + R) * (half ? 2 : 4), 'latent_rows');
    }
    this.cache = lender ? lender.cache : b.cache;
    const uk = new Uint16Array(H * D * C), ukT = new Uint16Array(H * C * D), uv = new Uint16Array(H * VD * C);
    placeRows(uk, C, 0, w.uk, H, d, D, rank);
    placeRows(uv, C, 0, w.uv, H, e, VD, rank);
    for (let h = 0; h < H; h++) {
      for (let r = 0; r < d; r++) for (let c = 0; c < rank; c++) ukT[(h * C + c) * D + r] = w.uk[(h * d + r) * rank + c];
    }
    b.wIn = upload(wIn, 'latent_in');
    b.wOut = upload(padOut(w.o, this.hidden, H, e, VD, this.k2), 'latent_out');
    b.uk = upload(half ? bf16ToF16(uk) : uk, 'latent_uk');
    b.uv = upload(half ? bf16ToF16(uv) : uv, 'latent_uv');
    b.ukT = upload(ukT, 'latent_uk_t');
    if (half) b.uvRows = upload(uv, 'latent_uv_rows');
    const tables = dec.rotary(m.rotBase, rot, rotaryTables);
    this.spec = packLatent({
      H, D, R, VD, rank, C, rotDim: rot, window: m.window, cacheDtype: half ? 'f16' : 'f32', dkvOffset: lender ? -1 : qRows, ldRow: this.ld, scale: m.scale,
      eps: this.eps, latentNorm: lender ? null : b.latentNorm, cos: tables.cos, sin: tables.sin, uk: b.uk, uv: b.uv, ukT: b.ukT, uvRows: half ? b.uvRows : b.uv,
    });
    this.workspace = getNative().latentDecodeWorkspaceBytes(this.spec, dec.config.maxSeq);
    dec.scratch('latent_decode', 1, this.workspace, 1);
    dec.scratch('row', this.ld, 1, 4);
    dec.scratch('mixed', this.k2, 1, 4);
  }

  step(recorder, pos, kvLen) {
    const d = this.dec, row = d.scratch('row', this.ld, 1, 4), mixed = d.scratch('mixed', this.k2, 1, 4);
    this.normedGemv(recorder, this.buffers.wIn, this.nIn, { output: row, nFirst: this.nIn });
    recordLatentDecode(recorder, this.spec, row, this.cache, mixed, pos, kvLen, d.config.maxSeq, d.scratch('latent_decode', 1, this.workspace, 1));
    this.outGemv(recorder, mixed, this.buffers.wOut, this.k2);
  }

  rows(recorder, x, count, pos) {
    const d = this.dec, normed = this.normedRows(recorder, x, count), rows = d.scratch('rows', this.ld, count, 4);
    this.inRows(recorder, normed, count, this.buffers.wIn, this.nIn, { output: rows, ldc: this.ld, nFirst: this.nIn });
    recordLatentRows(recorder, this.spec, rows, this.cache, count, pos);
    const mixed = d.scratch('mixed_rows', this.k2, count, d.operandBytes);
    const workspace = d.scratch('latent_prefill', 1, getNative().latentPrefillWorkspaceBytes(this.spec, count, pos), 1);
    recordLatentPrefill(recorder, this.spec, rows, this.cache, workspace, mixed, d.operand, this.k2, count, pos);
    this.outRows(recorder, mixed, this.k2, this.buffers.wOut, x, count);
  }
}

class MatrixMemory extends Sublayer {
  constructor(dec, m, w, norm, ls) {
    super(dec, norm, ls);
    const H = m.heads, d = m.dim, e = m.vdim, DP = up(d, 32), VP = up(e, 32), b = this.buffers;
    this.m = m;
    this.VP = VP;
    this.oWidth = H * VP;
    const at = { q: 0, k: H * DP, v: 2 * H * DP, g: 2 * H * DP + H * VP, i: 2 * H * (DP + VP), f: 2 * H * (DP + VP) + up(H, 4) };
    this.gOffset = at.g;
    this.nIn = at.f + up(H, 4);
    this.k2 = up(H * VP, 64);
    this.checkRow(Math.max(this.kx, this.k2));
    const wIn = new Uint16Array(this.nIn * this.kx), bias = new Float32Array(this.nIn), headNorm = new Float32Array(H * VP);
    for (const [name, size, padded] of [['q', d, DP], ['k', d, DP], ['v', e, VP], ['g', e, VP], ['i', 1, 1], ['f', 1, 1]]) {
      placeRows(wIn, this.kx, at[name], w[name], H, size, padded, this.hidden);
    }
    bias.set(w.iBias, at.i);
    bias.set(w.fBias, at.f);
    placeRows(headNorm, 1, 0, w.headNorm, H, e, VP, 1);
    b.wIn = upload(wIn, 'memory_in');
    b.bias = upload(bias, 'memory_bias');
    b.wOut = upload(padOut(w.o, this.hidden, H, e, VP, this.k2), 'memory_out');
    b.headNorm = upload(headNorm, 'head_norm');
    this.spec = packMlstm({ H, dim: d, vdim: e, DP, VP, kOffset: at.k, vOffset: at.v, iOffset: at.i, fOffset: at.f, ldRow: this.nIn, gateCap: m.gateCap });
    b.state = dec.zeroed(getNative().mlstmStateBytes(this.spec), 'memory_state');
    dec.scratch('row', this.nIn, 1, 4);
    dec.scratch('heads', this.oWidth, 1, 4);
    dec.scratch('mixed', this.k2, 1, 4);
  }

  get recurrent() {
    return true;
  }

  gateOf(rows) {
    return bufferWindow(rows, 4 * this.gOffset, rows.size - 4 * this.gOffset);
  }

  normGate(recorder, o, rows, output, dtype, count) {
    recordHeadNormGate(recorder, {
      input: o, ldIn: this.oWidth, gate: this.gateOf(rows), ldGate: this.nIn, headWeight: this.buffers.headNorm, output, dtype, ldOut: this.k2, rows: count,
      heads: this.m.heads, padded: this.VP, size: this.m.vdim, eps: this.eps,
    });
  }

  step(recorder, pos, kvLen) {
    const d = this.dec, b = this.buffers, row = d.scratch('row', this.nIn, 1, 4), o = d.scratch('heads', this.oWidth, 1, 4);
    this.normedGemv(recorder, b.wIn, this.nIn, { bias: b.bias, output: row, nFirst: this.nIn });
    recordMlstmStep(recorder, this.spec, row, b.state, o, pos, kvLen);
    if (this.m.heads <= GEMV_MAX_HEADS) {
      recordDenseGemvHeads(recorder, {
        input: o, gate: this.gateOf(row), headWeight: b.headNorm, heads: this.m.heads, padded: this.VP, size: this.m.vdim, eps: this.eps, weight: b.wOut,
        ldw: this.k2, N: this.hidden, K: this.k2, columnScale: b.ls, residual: d.step.x, output: d.step.x,
      });
      return;
    }
    const mixed = d.scratch('mixed', this.k2, 1, 4);
    this.normGate(recorder, o, row, mixed, 'f32', 1);
    this.outGemv(recorder, mixed, b.wOut, this.k2);
  }

  rows(recorder, x, count, pos) {
    const d = this.dec, b = this.buffers, normed = this.normedRows(recorder, x, count), rows = d.scratch('rows', this.nIn, count, 4);
    this.inRows(recorder, normed, count, b.wIn, this.nIn, { bias: b.bias, output: rows, ldc: this.nIn, nFirst: this.nIn });
    const o = d.scratch('heads_rows', this.oWidth, count, 4);
    const workspace = d.scratch('mlstm_prefill', 1, getNative().mlstmPrefillWorkspaceBytes(this.spec, count), 1);
    recordMlstmPrefill(recorder, this.spec, rows, b.state, workspace, o, this.oWidth, count, pos);
    const mixed = d.scratch('mixed_rows', this.k2, count, d.operandBytes);
    this.normGate(recorder, o, rows, mixed, d.operand, count);
    this.outRows(recorder, mixed, this.k2, b.wOut, x, count);
  }
}

class DenseFF extends Sublayer {
  constructor(dec, m, w, norm, ls) {
    super(dec, norm, ls);
    this.ff = m.ff;
    this.ffp = up(m.ff, 64);
    this.activation = m.activation;
    this.checkRow(Math.max(this.kx, this.ffp));
    const wUp = new Uint16Array(this.ff * this.kx);
    placeRows(wUp, this.kx, 0, w.up, 1, this.ff, this.ff, this.hidden);
    this.buffers.up = upload(wUp, 'ff_up');
    this.buffers.down = upload(padOut(w.down, this.hidden, 1, this.ff, this.ffp, this.ffp), 'ff_down');
    dec.scratch('act', this.ffp, 1, 4);
  }

  step(recorder) {
    const act = this.dec.scratch('act', this.ffp, 1, 4);
    this.normedGemv(recorder, this.buffers.up, this.ff, { nFirst: 0, output2: act, activation: this.activation });
    this.outGemv(recorder, act, this.buffers.down, this.ffp);
  }

  rows(recorder, x, count) {
    const d = this.dec, normed = this.normedRows(recorder, x, count), act = d.scratch('act_rows', this.ffp, count, d.operandBytes);
    this.inRows(recorder, normed, count, this.buffers.up, this.ff, { nFirst: 0, output2: act, ldc2: this.ffp, activation: this.activation });
    this.outRows(recorder, act, this.ffp, this.buffers.down, x, count);
  }
}

// gate and up rows [ff][n] into dst from row `at` on: 32 gate rows, the same 32 up rows, the next 32 gate rows, ..
function interleaveGateUp(dst, at, gate, upRows, ff, n, k) {
  for (let c = 0; c < ff; c++) {
    const row = at + 64 * (c >> 5) + (c & 31);
    dst.set(gate.subarray(c * n, (c + 1) * n), row * k);
    dst.set(upRows.subarray(c * n, (c + 1) * n), (row + 32) * k);
  }
}

class ExpertsFF extends Sublayer {
  constructor(dec, m, w, norm, ls) {
    super(dec, norm, ls);
    const E = m.experts, ff = m.ff, W = this.hidden, ffp = up(ff, 64), sfp = m.shared ? up(m.shared.ff, 64) : 0, b = this.buffers;
    this.checkRow(Math.max(this.kx, m.top * ffp + sfp));
    const router = new Uint16Array((E + (m.shared ? 1 : 0)) * this.kx);
    placeRows(router, this.kx, 0, w.router, 1, E, E, W);
    if (m.shared) router.set(w.sharedSg, E * this.kx);
    const wUp = new Uint16Array(E * 2 * ffp * this.kx), wDown = new Uint16Array(E * W * ffp);
    for (let j = 0; j < E; j++) {
      interleaveGateUp(wUp, j * 2 * ffp, w.gate[j], w.up[j], ff, W, this.kx);
      wDown.set(padOut(w.down[j], W, 1, ff, ffp, ffp), j * W * ffp);
    }
    b.router = upload(router, 'router');
    b.up = upload(wUp, 'experts_up');
    b.down = upload(wDown, 'experts_down');
    if (m.shared) {
      const sUp = new Uint16Array(2 * sfp * this.kx);
      interleaveGateUp(sUp, 0, w.sharedGate, w.sharedUp, m.shared.ff, W, this.kx);
      b.sharedUp = upload(sUp, 'shared_up');
      b.sharedDown = upload(padOut(w.sharedDown, W, 1, m.shared.ff, sfp, sfp), 'shared_down');
    }
    this.spec = packExperts({
      hidden: W, K: this.kx, experts: E, top: m.top, ff: ffp, sharedFf: sfp, eps: this.eps, limit: m.limit, sharedLimit: m.shared ? m.shared.limit : 0,
      norm: b.norm, layerScale: b.ls, router: b.router, up: b.up, down: b.down, sharedUp: b.sharedUp, sharedDown: b.sharedDown,
    });
    this.workspace = getNative().expertsStepWorkspaceBytes(this.spec);
    dec.scratch('experts_step', 1, this.workspace, 1);
  }

  step(recorder) {
    recordExpertsStep(recorder, this.spec, this.dec.step.x, this.dec.scratch('experts_step', 1, this.workspace, 1));
  }

  rows(recorder, x, count) {
    const d = this.dec, normed = this.normedRows(recorder, x, count);
    const workspace = d.scratch('experts_prefill', 1, getNative().expertsPrefillWorkspaceBytes(this.spec, DTYPE[d.operand], count), 1);
    recordExpertsPrefill(recorder, this.spec, normed, d.operand, x, this.kx, workspace, count);
  }
}

const MIXERS = { latent_attention: LatentAttention, mlstm: MatrixMemory };
const FEED_FORWARDS = { dense: DenseFF, experts: ExpertsFF };

export class SequentialLayer {
  // spec: {mixer: {type, ..}, mlp: {type, ..} | null}; w: {norm1, ls1, mixer, norm2, ls2, mlp}; earlier: the layers so far
  constructor(dec, spec, w, earlier) {
    const lender = spec.mixer.kvFrom === null || spec.mixer.kvFrom === undefined ? null : earlier[spec.mixer.kvFrom].mixer;
    this.mixer = new MIXERS[spec.mixer.type](dec, spec.mixer, w.mixer, w.norm1, w.ls1, lender);
    this.parts = [this.mixer];
    if (spec.mlp) this.parts.push(new FEED_FORWARDS[spec.mlp.type](dec, spec.mlp, w.mlp, w.norm2, w.ls2));
  }

  get recurrent() {
    return this.parts.some((p) => p.recurrent === true);
  }

  step(recorder, pos, kvLen) {
    for (const p of this.parts) p.step(recorder, pos, kvLen);
  }

  rows(recorder, x, count, pos) {
    for (const p of this.parts) p.rows(recorder, x, count, pos);
  }

  ownBuffers() {
    return [].concat(...this.parts.map((p) => Object.values(p.buffers)));
  }
}
