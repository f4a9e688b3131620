// The Qwen3-class Q4_K model over the HIP op API: the ops of the reference's decodeStep
// (src/inference/pipelines/text/generator-steps.js:588-820), recorded in execution-graph order
// (src/config/conversion/qwen3/qwen-3-embedding-0-6b-q4k-ehf16-af32.json `execution.decode`).
// The loops around them are TextDecoder's.
import {
  createTensor, createWeightBuffer, acquireBuffer, releaseBuffer,
  recordGather, recordRMSNorm, recordMatmul, recordSplitQKVRMSNormRoPEQK,
  recordAttention, recordFusedNormedFFN, recordFusedFFN, recordLmHeadArgmaxF16, lmHeadArgmaxNormFusable,
  recordDecodeAttentionFromQKV, decodeAttentionFromQKVSupported,
  recordLayerChain, recordDecodeAttentionPartials, layerChainSupported, layerChainMergesAttention,
  recordCheckFiniteness,
} from '../kernel-selector.js';
import { TextDecoder, FinitenessError, bufferWindow, upload } from './text-decoder.js';

export { FinitenessError };

export class HipTextDecoder extends TextDecoder {
  // config: {layers, hidden, inter, heads, kvHeads, headDim, vocab, eps, maxSeq}
  //   finitenessGuard, finitenessAbsThreshold: see TextDecoder
  // weights: {layers: [{wqkv, wo, wgate, wup, wdown (Uint8Array Q4_K), inputNorm, postAttnNorm,
  //           qNorm, kNorm (Float32Array)}], embed (Uint16Array f16 bits), finalNorm, cos, sin}
  constructor(config, weights) {
    super(config);
    const c = config;
    this.qSize = c.heads * c.headDim;
    this.kSize = c.kvHeads * c.headDim;
    this.layers = weights.layers.map((l, i) => ({
      wqkv: createWeightBuffer(upload(l.wqkv, `L${i}.qkv`), 'q4k', 'row', [this.qSize + 2 * this.kSize, c.hidden], `L${i}.qkv`),
      wo: createWeightBuffer(upload(l.wo, `L${i}.o`), 'q4k', 'row', [c.hidden, this.qSize], `L${i}.o`),
      wgate: createWeightBuffer(upload(l.wgate, `L${i}.gate`), 'q4k', 'row', [c.inter, c.hidden], `L${i}.gate`),
      wup: createWeightBuffer(upload(l.wup, `L${i}.up`), 'q4k', 'row', [c.inter, c.hidden], `L${i}.up`),
      wdown: createWeightBuffer(upload(l.wdown, `L${i}.down`), 'q4k', 'row', [c.hidden, c.inter], `L${i}.down`),
      inputNorm: createTensor(upload(l.inputNorm), 'f32', [c.hidden], 'input_norm'),
      postAttnNorm: createTensor(upload(l.postAttnNorm), 'f32', [c.hidden], 'post_attn_norm'),
      qNorm: createTensor(upload(l.qNorm), 'f32', [c.headDim], 'q_norm'),
      kNorm: createTensor(upload(l.kNorm), 'f32', [c.headDim], 'k_norm'),
      cacheK: createTensor(acquireBuffer(c.maxSeq * this.kSize * 2, undefined, 'kv_k'), 'f16', [c.maxSeq, c.kvHeads, c.headDim], 'kv_k'),
      cacheV: createTensor(acquireBuffer(c.maxSeq * this.kSize * 2, undefined, 'kv_v'), 'f16', [c.maxSeq, c.kvHeads, c.headDim], 'kv_v'),
    }));
    this.embed = createWeightBuffer(upload(weights.embed, 'embed'), 'f16', 'row', [c.vocab, c.hidden], 'embed');
    this.finalNorm = createTensor(upload(weights.finalNorm), 'f32', [c.hidden], 'final_norm');
    this.cos = createTensor(upload(weights.cos), 'f32', [c.maxSeq, c.headDim / 2], 'rope_cos');
    this.sin = createTensor(upload(weights.sin), 'f32', [c.maxSeq, c.headDim / 2], 'rope_sin');
    // decode steps: q/k norm, RoPE and the KV append run inside the attention kernel when the head
    // geometry allows it (one launch fewer per layer)
    this.fuseQkvAttention = config.fuseQkvAttention !== false &&
      decodeAttentionFromQKVSupported(c.heads, c.kvHeads, c.headDim, c.headDim, false);
    // ... and the products between two attentions go out as one chained launch that also merges the
    // attention's key splits (two launches per layer), where the shapes are served and the guard is off
    this.chainGemvs = config.chainGemvs !== false && this.fuseQkvAttention && config.finitenessGuard !== true &&
      layerChainSupported(c.hidden, c.inter, this.qSize) && layerChainMergesAttention(c.heads, c.kvHeads, c.headDim, c.maxSeq);
  }

  deviceKvLenServed() {
    return this.fuseQkvAttention;
  }

  // Final RMSNorm + LM head + argmax of one hidden row: one launch with the norm inside the LM head kernel
  // where the hidden size allows it, else the norm as a launch of its own in front.
  async recordNormedLmHead(recorder, temps, hiddenRow, tokenOut, tokenIndex, logitsOutput) {
    const c = this.config;
    const opts = { vocabSize: c.vocab, hiddenSize: c.hidden, outputBuffer: tokenOut, outputIndex: tokenIndex, logitsOutput };
    if (lmHeadArgmaxNormFusable(c.hidden)) {
      await recordLmHeadArgmaxF16(recorder, hiddenRow, this.embed, Object.assign({ normWeight: this.finalNorm, rmsNormEps: c.eps }, opts));
      return;
    }
    const normed = await recordRMSNorm(recorder, hiddenRow, this.finalNorm, c.eps, { batchSize: 1, hiddenSize: c.hidden });
    temps.push(normed.buffer);
    await recordLmHeadArgmaxF16(recorder, normed, this.embed, opts);
  }

  // A portion through the batched path: prefill GEMMs + prefill attention.
  async recordPrefillChunk(recorder, temps, ids, part, pos) {
    const c = this.config, T = part.length;
    const temp = (t) => { temps.push(t.buffer); return t; };
    let x = temp(await recordGather(recorder, bufferWindow(ids, 4, 4 * T), this.embed, T, c.hidden, c.vocab, { embeddingDtype: 'f16', outputDtype: 'f32' }));
    for (let li = 0; li < this.layers.length; li++) {
      const l = this.layers[li];
      // the input RMSNorm runs inside the product (GEMV prologue below 16 tokens, the GEMM's activation
      // packing from 16 on) unless the model asks for separate norm launches
      const fusedNorm = c.fuseNorm !== false;
      let qkv;
      if (fusedNorm) {
        qkv = temp(await recordMatmul(recorder, x, l.wqkv, T, this.qSize + 2 * this.kSize, c.hidden,
          { outputDtype: 'f32', role: 'qkv_proj', layerIdx: li,
            normWeight: l.inputNorm, rmsNormEps: c.eps, useFusedRmsnormWideTile: true }));
      } else {
        const normed = temp(await recordRMSNorm(recorder, x, l.inputNorm, c.eps, { batchSize: T, hiddenSize: c.hidden }));
        qkv = temp(await recordMatmul(recorder, normed, l.wqkv, T, this.qSize + 2 * this.kSize, c.hidden,
          { outputDtype: 'f32', role: 'qkv_proj', layerIdx: li }));
      }
      const split = await recordSplitQKVRMSNormRoPEQK(recorder, qkv, l.qNorm, l.kNorm, this.cos, this.sin, c.eps, {
        numTokens: T, numHeads: c.heads, numKVHeads: c.kvHeads, headDim: c.headDim,
        qSize: this.qSize, kSize: this.kSize, vSize: this.kSize, startPos: pos,
        f16KVCacheWrite: { keysBuffer: l.cacheK.buffer, valuesBuffer: l.cacheV.buffer, dstOffset: pos * this.kSize },
      });
      temp(split.Q);
      const attn = temp(await recordAttention(recorder, split.Q, l.cacheK, l.cacheV, null, c.heads, c.headDim, {
        seqLen: T, kvLen: pos + T, numKVHeads: c.kvHeads, causal: true, startPos: pos, layerIdx: li,
      }));
      const attnFlat = createTensor(attn.buffer, 'f32', [T, this.qSize], 'attn_flat');
      const x2 = temp(await recordMatmul(recorder, attnFlat, l.wo, T, c.hidden, this.qSize,
        { outputDtype: 'f32', role: 'o_proj', layerIdx: li, residualTensor: x }));
      let act;
      if (fusedNorm) {
        act = temp(await recordFusedNormedFFN(recorder, x2, l.postAttnNorm, c.eps, l.wgate, l.wup, c.hidden, c.inter,
          { batchSize: T, activation: 'silu' }));
      } else {
        const normed2 = temp(await recordRMSNorm(recorder, x2, l.postAttnNorm, c.eps, { batchSize: T, hiddenSize: c.hidden }));
        act = temp(await recordFusedFFN(recorder, normed2, l.wgate, l.wup, c.hidden, c.inter,
          { batchSize: T, activation: 'silu' }));
      }
      x = temp(await recordMatmul(recorder, act, l.wdown, T, c.hidden, c.inter,
        { outputDtype: 'f32', role: 'down_proj', layerIdx: li, residualTensor: x2 }));
    }
    return { buffer: x.buffer, rowFloats: c.hidden };
  }

  async recordEmbedding(recorder, temps, ids, prev, pos, options) {
    const c = this.config;
    const x = await recordGather(recorder, ids, this.embed, 1, c.hidden, c.vocab, { embeddingDtype: 'f16', outputDtype: 'f32' });
    temps.push(x.buffer);
    return x;
  }

  async recordLayers(recorder, temps, x, pos, options) {
    const c = this.config;
    const temp = (t) => { temps.push(t.buffer); return t; };
    if (this.chainGemvs) return this.recordChainedLayers(recorder, temps, x, pos, options);
    for (let li = 0; li < this.layers.length; li++) {
      const l = this.layers[li];
      // input RMSNorm runs in the prologue of the stacked q/k/v projection
      const qkv = temp(await recordMatmul(recorder, x, l.wqkv, 1, this.qSize + 2 * this.kSize, c.hidden,
        { outputDtype: 'f32', role: 'qkv_proj', layerIdx: li,
          normWeight: l.inputNorm, rmsNormEps: c.eps, useFusedRmsnormWideTile: true }));
      let attn;
      if (this.fuseQkvAttention) {
        attn = temp(await recordDecodeAttentionFromQKV(recorder, qkv, l.qNorm, l.kNorm, this.cos, this.sin, c.eps,
          l.cacheK, l.cacheV, { numHeads: c.heads, numKVHeads: c.kvHeads, headDim: c.headDim, startPos: pos, layerIdx: li,
            // a captured step reads the key count from the word behind the token id, so a replay needs no patching
            kvLenBuffer: options.deviceKvLen ? bufferWindow(this.ids, 4, 4) : null, maxKvLen: c.maxSeq }));
      } else {
        const split = await recordSplitQKVRMSNormRoPEQK(recorder, qkv, l.qNorm, l.kNorm, this.cos, this.sin, c.eps, {
          numTokens: 1, numHeads: c.heads, numKVHeads: c.kvHeads, headDim: c.headDim,
          qSize: this.qSize, kSize: this.kSize, vSize: this.kSize, startPos: pos,
          f16KVCacheWrite: { keysBuffer: l.cacheK.buffer, valuesBuffer: l.cacheV.buffer, dstOffset: pos * this.kSize },
        });
        temp(split.Q);
        attn = temp(await recordAttention(recorder, split.Q, l.cacheK, l.cacheV, null, c.heads, c.headDim, {
          seqLen: 1, kvLen: pos + 1, numKVHeads: c.kvHeads, causal: true, startPos: pos, layerIdx: li,
        }));
      }
      const attnFlat = createTensor(attn.buffer, 'f32', [1, this.qSize], 'attn_flat');
      const x2 = temp(await recordMatmul(recorder, attnFlat, l.wo, 1, c.hidden, this.qSize,
        { outputDtype: 'f32', role: 'o_proj', layerIdx: li, residualTensor: x }));
      const act = temp(await recordFusedNormedFFN(recorder, x2, l.postAttnNorm, c.eps, l.wgate, l.wup, c.hidden, c.inter,
        { batchSize: 1, activation: 'silu' }));
      x = temp(await recordMatmul(recorder, act, l.wdown, 1, c.hidden, c.inter,
        { outputDtype: 'f32', role: 'down_proj', layerIdx: li, residualTensor: x2 }));
      if (this.finitenessGuard) {
        recordCheckFiniteness(recorder, x, c.hidden, this.finitenessStatus, li, pos, this.finitenessAbsThreshold);
      }
    }
    return x;
  }

  // The layers of a decode step at two launches each: the attention's split kernel, then one chained
  // launch that merges the splits and runs o + residual, RMSNorm + gate/up + SiLU, down + residual and
  // the next layer's RMSNorm + q/k/v.  Returns the last layer's output row.
  async recordChainedLayers(recorder, temps, x, pos, options) {
    const c = this.config;
    const qkvSize = this.qSize + 2 * this.kSize;
    const f32 = (n, label) => { const b = acquireBuffer(n * 4, undefined, label); temps.push(b); return b; };
    const l0 = this.layers[0];
    let qkv = await recordMatmul(recorder, x, l0.wqkv, 1, qkvSize, c.hidden,
      { outputDtype: 'f32', role: 'qkv_proj', layerIdx: 0, normWeight: l0.inputNorm, rmsNormEps: c.eps, useFusedRmsnormWideTile: true });
    temps.push(qkv.buffer);
    let xb = x.buffer;
    for (let li = 0; li < this.layers.length; li++) {
      const l = this.layers[li];
      const next = li + 1 < this.layers.length ? this.layers[li + 1] : null;
      const attention = recordDecodeAttentionPartials(recorder, qkv, l.qNorm, l.kNorm, this.cos, this.sin, c.eps, l.cacheK, l.cacheV, {
        numHeads: c.heads, numKVHeads: c.kvHeads, headDim: c.headDim, startPos: pos,
        kvLenBuffer: options.deviceKvLen ? bufferWindow(this.ids, 4, 4) : null, maxKvLen: c.maxSeq,
      });
      temps.push(attention.workspace);
      const x2 = f32(c.hidden, 'attn_output'), act = f32(c.inter, 'ffn_act'), xOut = f32(c.hidden, 'layer_output');
      const phases = [
        { weight: l.wo, output: x2, residual: xb, N: c.hidden, K: this.qSize },
        { weight: l.wgate, weight2: l.wup, output: act, normWeight: l.postAttnNorm, N: c.inter, K: c.hidden, activation: 'silu', rmsNormEps: c.eps },
        { weight: l.wdown, output: xOut, residual: x2, N: c.hidden, K: c.inter },
      ];
      let qkvNext = null;
      if (next) {
        qkvNext = f32(qkvSize, 'qkv');
        phases.push({ weight: next.wqkv, output: qkvNext, normWeight: next.inputNorm, N: qkvSize, K: c.hidden, rmsNormEps: c.eps });
      }
      recordLayerChain(recorder, null, phases, attention);
      xb = xOut;
      if (next) qkv = createTensor(qkvNext, 'f32', [1, qkvSize], 'qkv');
    }
    return createTensor(xb, 'f32', [1, c.hidden], 'layer_output');
  }

  releaseWeights() {
    for (const l of this.layers) {
      for (const key of Object.keys(l)) releaseBuffer(l[key].buffer);
    }
  }
}
