// Ops of models with dense bf16 weights (no counterpart in the reference's Q4_K path): embedding sums, row norms into
// the operand type, the stacked products with two outputs, and attention with a distance bias, value norm and
// head gates.  Buffers are caller-provided; the C ABI checks the shapes (include/doppler_hip.h).
import { getNative, DTYPE, DENSE_ACT } from '../native.js';
import { acquireBuffer } from '../buffer-pool.js';
import { bufferOf, noteDispatch } from './constants.js';

const SPEC_BYTES = 72;       // struct dh_attn_spec

function ptr(x) {
  return x === null || x === undefined ? null : bufferOf(x).ptr;
}

function need(op, name, x, bytes) {
  const b = bufferOf(x);
  if (b.size < bytes) throw new Error(`[${op}] ${name} buffer smaller than ${bytes} bytes (${b.size}).`);
}

function code(op, table, key) {
  if (!(key in table)) throw new Error(`[${op}] unknown ${table === DTYPE ? 'dtype' : 'activation'} "${key}".`);
  return table[key];
}

// options: {ids, indexOffset, prev, embed, vocab, bigram: {table, buckets, mulPrev, mulCur}|null, pos: {table, count}|null,
//           output, ldOut, numTokens, hidden, startPos, kvLenBuffer}
export function recordEmbedSum(recorder, o) {
  need('EmbedSum', 'embedding', o.embed, o.vocab * o.hidden * 2);
  need('EmbedSum', 'output', o.output, ((o.numTokens - 1) * o.ldOut + o.hidden) * 4);
  if (o.bigram) need('EmbedSum', 'bigram', o.bigram.table, (o.bigram.buckets + 1) * o.hidden * 2);
  if (o.pos) need('EmbedSum', 'position', o.pos.table, o.pos.count * o.hidden * 2);
  getNative().embedSum(ptr(o.ids), o.indexOffset || 0, ptr(o.prev), ptr(o.embed), o.vocab, o.bigram ? ptr(o.bigram.table) : null,
    o.bigram ? o.bigram.buckets : 0, o.bigram ? o.bigram.mulPrev : 0, o.bigram ? o.bigram.mulCur : 0, o.pos ? ptr(o.pos.table) : null,
    o.pos ? o.pos.count : 0, ptr(o.output), o.ldOut, o.numTokens, o.hidden, o.startPos, ptr(o.kvLenBuffer));
  noteDispatch(recorder, 'embed_sum');
}

// options: {input, ldIn, rows, weight, output, dtype, ldOut, count, hidden, eps}
export function recordRMSNormRows(recorder, o) {
  need('RMSNormRows', 'weight', o.weight, o.hidden * 4);
  need('RMSNormRows', 'output', o.output, o.count * o.ldOut * (o.dtype === 'bf16' ? 2 : 4));
  getNative().rmsnormRows(ptr(o.input), o.ldIn, ptr(o.rows), ptr(o.weight), ptr(o.output), code('RMSNormRows', DTYPE, o.dtype), o.ldOut,
    o.count, o.hidden, o.eps);
  noteDispatch(recorder, 'rmsnorm_rows');
}

// options: {input, dtype, lda, weight, ldw, M, N, K, alpha, bias, residual, output, ldc, nFirst, output2, dtype2, ldc2, activation}
export function recordDenseMatmul(recorder, o) {
  need('DenseMatmul', 'weight', o.weight, o.N * o.ldw * 2);
  need('DenseMatmul', 'input', o.input, ((o.M - 1) * o.lda + o.K) * (o.dtype === 'bf16' ? 2 : 4));
  getNative().denseMatmul(ptr(o.input), code('DenseMatmul', DTYPE, o.dtype), o.lda, ptr(o.weight), o.ldw, o.M, o.N, o.K,
    o.alpha === undefined ? 1.0 : o.alpha, ptr(o.bias), ptr(o.residual), ptr(o.output), o.ldc, o.nFirst, ptr(o.output2),
    o.output2 ? code('DenseMatmul', DTYPE, o.dtype2) : 0, o.ldc2 || 0, code('DenseMatmul', DENSE_ACT, o.activation || 'none'));
  noteDispatch(recorder, 'dense_matmul');
}

// options: {input, normWeight, hidden, eps, weight, ldw, N, K, alpha, bias, residual, output, nFirst, output2, activation}
export function recordDenseGemv(recorder, o) {
  need('DenseGemv', 'weight', o.weight, o.N * o.ldw * 2);
  need('DenseGemv', 'input', o.input, o.K * 4);
  if (o.normWeight) need('DenseGemv', 'norm weight', o.normWeight, o.K * 4);
  getNative().denseGemv(ptr(o.input), ptr(o.normWeight), o.hidden || 0, o.eps || 0, ptr(o.weight), o.ldw, o.N, o.K,
    o.alpha === undefined ? 1.0 : o.alpha, ptr(o.bias), ptr(o.residual), ptr(o.output), o.nFirst, ptr(o.output2),
    code('DenseGemv', DENSE_ACT, o.activation || 'none'));
  noteDispatch(recorder, 'dense_gemv');
}

// options: {input, normWeight, hidden, eps, weight, ldw, vocab, K, alpha, outputBuffer, outputIndex, logitsOutput}
export function recordDenseLmHeadArgmax(recorder, o) {
  need('DenseLmHead', 'weight', o.weight, o.vocab * o.ldw * 2);
  need('DenseLmHead', 'input', o.input, o.K * 4);
  need('DenseLmHead', 'output', o.outputBuffer, 4 * ((o.outputIndex || 0) + 1));
  if (o.logitsOutput) need('DenseLmHead', 'logits', o.logitsOutput, o.vocab * 4);
  const native = getNative();
  const workspace = acquireBuffer(native.lmheadArgmaxWorkspaceBytes(o.vocab), undefined, 'lm_head_argmax_temp');
  recorder.trackTemporaryBuffer(workspace);
  native.denseLmheadArgmax(ptr(o.input), ptr(o.normWeight), o.hidden, o.eps, ptr(o.weight), o.ldw, o.vocab, o.K,
    o.alpha === undefined ? 1.0 : o.alpha, workspace.ptr, ptr(o.outputBuffer), o.outputIndex || 0, ptr(o.logitsOutput));
  noteDispatch(recorder, 'dense_lm_head_argmax');
}

// s: {heads, kvHeads, D, VD, valueDim, window, cacheDtype, valueNorm, kOffset, vOffset, gateOffset, ldQkv, scale, valueEps,
//     biasR1, biasR2}
export function packAttnSpec(s) {
  const bytes = getNative().attnSpecBytes();
  if (bytes !== SPEC_BYTES) throw new Error(`[AttnSpec] struct size of the library (${bytes}) differs from this host's (${SPEC_BYTES}).`);
  const v = new DataView(new ArrayBuffer(SPEC_BYTES));
  [s.heads, s.kvHeads, s.D, s.VD, s.valueDim, s.window, code('AttnSpec', DTYPE, s.cacheDtype), s.valueNorm ? 1 : 0, s.kOffset, s.vOffset,
    s.gateOffset, s.ldQkv].forEach((x, i) => v.setInt32(4 * i, x, true));
  v.setFloat32(48, s.scale, true);
  v.setFloat32(52, s.valueEps, true);
  v.setBigUint64(56, s.biasR1 ? ptr(s.biasR1) : 0n, true);
  v.setBigUint64(64, s.biasR2 ? ptr(s.biasR2) : 0n, true);
  return new Uint8Array(v.buffer);
}

export function recordAttnSpecKVWrite(recorder, spec, qkv, cacheK, cacheV, numTokens, startPos) {
  getNative().attnSpecKvWrite(spec, ptr(qkv), ptr(cacheK), ptr(cacheV), numTokens, startPos);
  noteDispatch(recorder, 'attn_spec_kv_write');
}

export function recordAttnSpecPrefill(recorder, spec, qkv, cacheK, cacheV, output, dtype, ldOut, numTokens, startPos) {
  getNative().attnSpecPrefill(spec, ptr(qkv), ptr(cacheK), ptr(cacheV), ptr(output), code('AttnSpec', DTYPE, dtype), ldOut, numTokens, startPos);
  noteDispatch(recorder, 'attn_spec_prefill');
}

// kvLenBuffer: device word with the key count pos + 1, at most maxKvLen (captured steps), or null
export function recordAttnSpecDecode(recorder, spec, qkv, cacheK, cacheV, output, pos, kvLenBuffer, maxKvLen, workspace) {
  getNative().attnSpecDecode(spec, ptr(qkv), ptr(cacheK), ptr(cacheV), ptr(output), pos, ptr(kvLenBuffer), maxKvLen, ptr(workspace));
  noteDispatch(recorder, 'attn_spec_decode');
}
