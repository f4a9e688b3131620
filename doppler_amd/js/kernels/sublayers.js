// Ops of sequential layers (latent attention, matrix memory, mixtures of experts; include/doppler_hip.h).  Specs are packed
// once per layer into the bytes of their C structs; the C ABI checks the shapes.
import { getNative, DTYPE, DENSE_ACT } from '../native.js';
import { bufferOf, noteDispatch } from './constants.js';

const ptr = (x) => (x === null || x === undefined ? null : bufferOf(x).ptr);

// fields: ['int' | 'float' | 'ptr', value] in the order of the C struct `name`
function pack(name, fields) {
  const expected = getNative().sublayerStructBytes()[['latent', 'mlstm', 'experts'].indexOf(name)];
  const v = new DataView(new ArrayBuffer(expected + 8));
  let at = 0;
  for (const [kind, value] of fields) {
    if (kind === 'ptr') {
      at = Math.ceil(at / 8) * 8;
      v.setBigUint64(at, value ? ptr(value) : 0n, true);
      at += 8;
    } else {
      if (kind === 'int') v.setInt32(at, value, true);
      else v.setFloat32(at, value, true);
      at += 4;
    }
  }
  if (at !== expected) throw new Error(`[${name}] struct size of the library (${expected}) differs from this host's (${at}).`);
  return new Uint8Array(v.buffer, 0, expected);
}

const ints = (...values) => values.map((x) => ['int', x]);
const floats = (...values) => values.map((x) => ['float', x]);
const ptrs = (...values) => values.map((x) => ['ptr', x]);

export function packLatent(s) {
  return pack('latent', [].concat(
    ints(s.H, s.D, s.R, s.VD, s.rank, s.C, s.rotDim, s.window, DTYPE[s.cacheDtype], s.dkvOffset, s.ldRow), floats(s.scale, s.eps),
    ptrs(s.latentNorm, s.cos, s.sin, s.uk, s.uv, s.ukT, s.uvRows)));
}

export function packMlstm(s) {
  return pack('mlstm', [].concat(ints(s.H, s.dim, s.vdim, s.DP, s.VP, s.kOffset, s.vOffset, s.iOffset, s.fOffset, s.ldRow), floats(s.gateCap)));
}

export function packExperts(s) {
  return pack('experts', [].concat(ints(s.hidden, s.K, s.experts, s.top, s.ff, s.sharedFf), floats(s.eps, s.limit, s.sharedLimit),
    ptrs(s.norm, s.layerScale, s.router, s.up, s.down, s.sharedUp, s.sharedDown)));
}

// options: {input, dtype, lda, weight, ldw, M, N, K, bias, columnScale, residual, output, ldc, nFirst, output2, ldc2, activation}
export function recordDenseMatmulScaled(recorder, o) {
  getNative().denseMatmulScaled(ptr(o.input), DTYPE[o.dtype], o.lda, ptr(o.weight), o.ldw, o.M, o.N, o.K, 1.0, ptr(o.bias), ptr(o.columnScale),
    ptr(o.residual), ptr(o.output), o.ldc || 0, o.nFirst, ptr(o.output2), DTYPE[o.dtype], o.ldc2 || 0, DENSE_ACT[o.activation || 'none']);
  noteDispatch(recorder, 'dense_matmul');
}

// options: {input, normWeight, hidden, eps, weight, ldw, N, K, bias, columnScale, residual, output, nFirst, output2, activation}
export function recordDenseGemvScaled(recorder, o) {
  getNative().denseGemvScaled(ptr(o.input), ptr(o.normWeight), o.hidden || 0, o.eps || 0, ptr(o.weight), o.ldw, o.N, o.K, 1.0, ptr(o.bias),
    ptr(o.columnScale), ptr(o.residual), ptr(o.output), o.nFirst, ptr(o.output2), DENSE_ACT[o.activation || 'none']);
  noteDispatch(recorder, 'dense_gemv');
}

// options: {input, gate, headWeight, heads, padded, size, eps, weight, ldw, N, K, columnScale, residual, output}
export function recordDenseGemvHeads(recorder, o) {
  getNative().denseGemvHeads(ptr(o.input), ptr(o.gate), ptr(o.headWeight), o.heads, o.padded, o.size, o.eps, ptr(o.weight), o.ldw, o.N, o.K,
    ptr(o.columnScale), ptr(o.residual), ptr(o.output));
  noteDispatch(recorder, 'dense_gemv_heads');
}

// options: {input, ldIn, gate, ldGate, headWeight, output, dtype, ldOut, rows, heads, padded, size, eps}
export function recordHeadNormGate(recorder, o) {
  getNative().headNormGate(ptr(o.input), o.ldIn, ptr(o.gate), o.ldGate, ptr(o.headWeight), ptr(o.output), DTYPE[o.dtype], o.ldOut, o.rows, o.heads,
    o.padded, o.size, o.eps);
  noteDispatch(recorder, 'head_norm_gate');
}

export function recordLatentRows(recorder, spec, rows, cache, numTokens, startPos) {
  getNative().latentRows(spec, ptr(rows), ptr(cache), numTokens, startPos);
  noteDispatch(recorder, 'latent_rows');
}

export function recordLatentPrefill(recorder, spec, rows, cache, workspace, output, dtype, ldOut, numTokens, startPos) {
  getNative().latentPrefill(spec, ptr(rows), ptr(cache), ptr(workspace), ptr(output), DTYPE[dtype], ldOut, numTokens, startPos);
  noteDispatch(recorder, 'latent_prefill');
}

// kvLenBuffer as in recordAttnSpecDecode
export function recordLatentDecode(recorder, spec, row, cache, output, pos, kvLenBuffer, maxKvLen, workspace) {
  getNative().latentDecode(spec, ptr(row), ptr(cache), ptr(output), pos, ptr(kvLenBuffer), maxKvLen, ptr(workspace));
  noteDispatch(recorder, 'latent_decode');
}

export function recordMlstmStep(recorder, spec, row, state, output, pos, kvLenBuffer) {
  getNative().mlstmStep(spec, ptr(row), ptr(state), ptr(output), pos, ptr(kvLenBuffer));
  noteDispatch(recorder, 'mlstm_step');
}

export function recordMlstmPrefill(recorder, spec, rows, state, workspace, output, ldOut, numTokens, startPos) {
  getNative().mlstmPrefill(spec, ptr(rows), ptr(state), ptr(workspace), ptr(output), ldOut, numTokens, startPos);
  noteDispatch(recorder, 'mlstm_prefill');
}

export function recordExpertsStep(recorder, spec, residual, workspace) {
  getNative().expertsStep(spec, ptr(residual), ptr(workspace));
  noteDispatch(recorder, 'experts_step');
}

export function recordExpertsPrefill(recorder, spec, normed, dtype, residual, ldResidual, workspace, numTokens) {
  getNative().expertsPrefill(spec, ptr(normed), DTYPE[dtype], ptr(residual), ldResidual, ptr(workspace), numTokens);
  noteDispatch(recorder, 'experts_prefill');
}
