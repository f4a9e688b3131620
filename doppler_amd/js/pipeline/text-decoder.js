// Generation over a step a model records: decode steps with one 4-byte readback per token, the staged greedy loop,
// captured steps, prompts in portions, sampling.  The shape of the reference's decodeStep
// (src/inference/pipelines/text/generator-steps.js:588-820): one CommandRecorder per token, one readback.
//
// A model (subclass) provides
//   recordEmbedding(recorder, temps, ids, prev, pos, options)   the step's residual row (tensor); ids and prev are device
//                                                               words with the token and the one before it
//   recordLayers(recorder, temps, x, pos, options)              its layers; returns the final residual row
//   recordNormedLmHead(recorder, temps, row, tokenOut, tokenIndex, logitsOutput)
//   recordPrefillChunk(recorder, temps, ids, part, pos)         a portion; returns its final residual rows
//                                                               {buffer, rowFloats}; ids: device words [before, part...]
//   deviceKvLenServed()                                         whether captured steps read the key count on the device
//   carriesState()                                              whether its layers carry recurrent state: positions must then follow
//                                                               one another, or start again at 0
//   releaseWeights()
import {
  createTensor, acquireBuffer, releaseBuffer, uploadData, readBufferSlice, createCommandRecorder, recordGPUSample,
  parseFinitenessStatusWords, resolveFinitenessAbsThreshold, FINITENESS_STATUS_BYTES,
} from '../kernel-selector.js';
import { getNative } from '../native.js';

// A window of a device buffer starting `offset` bytes in (no ownership: never released).
export function bufferWindow(buffer, offset, size) {
  return { ptr: buffer.ptr + BigInt(offset), size, capacity: size, label: buffer.label };
}

// An activation left the f16 range (or the configured bound) during a decode step
// (reference: src/inference/pipelines/text/generator-steps.js:164-169).
export class FinitenessError extends Error {
  constructor(message) {
    super(message);
    this.name = 'FinitenessError';
  }
}

export function upload(bytes, label) {
  const buf = acquireBuffer(bytes.byteLength, undefined, label);
  uploadData(buf, bytes);
  return buf;
}

// decodeGreedy: tokens in flight between the device and the host (ring slots), and the events that mark
// their copies
const TOKEN_RING = 64;
const READ_EVENTS = 4;

export class TextDecoder {
  // config: {vocab, maxSeq, ...}
  //   finitenessGuard (default false): check every layer's output against finitenessAbsThreshold
  //   (one more launch per layer) and read the status words back beside the token, as the
  //   reference does for f16 activations (layer.js:1237-1252, generator-steps.js:786-798, :837-843)
  constructor(config) {
    this.config = config;
    // the step's token id, its key count (captured steps), the token before it
    this.ids = acquireBuffer(16, undefined, 'token_ids');
    // [token, status, layer, step, pad]: the staging layout of the reference's guarded readback
    this.tokenOut = acquireBuffer(4 + FINITENESS_STATUS_BYTES, undefined, 'sampled_token');
    this.finitenessGuard = config.finitenessGuard === true;
    this.finitenessAbsThreshold = resolveFinitenessAbsThreshold(config.finitenessAbsThreshold);
    this.finitenessStatus = bufferWindow(this.tokenOut, 4, FINITENESS_STATUS_BYTES);
    this.logits = null;
    this.readback = null;
    // tokens fed so far by position: a model whose embedding reads the previous token finds it here
    this.history = new Uint32Array(config.maxSeq);
    this.statePos = 0;     // the position recurrent state is ready for
  }

  carriesState() {
    return false;
  }

  advance(pos, tokens) {
    if (pos !== 0 && pos !== this.statePos && this.carriesState()) {
      throw new Error(`the sequence's recurrent state stands at position ${this.statePos}, not at ${pos}`);
    }
    this.statePos = pos + tokens;
  }

  remember(pos, tokens) {
    for (let i = 0; i < tokens.length && pos + i < this.history.length; i++) this.history[pos + i] = tokens[i];
  }

  tokenBefore(pos) {
    return pos > 0 ? this.history[pos - 1] : 0;
  }

  uploadStep(token, pos, kvLen = 0) {
    uploadData(this.ids, new Uint32Array([token, kvLen, this.tokenBefore(pos)]));
    this.remember(pos, [token]);
  }

  // Output head of one hidden row; greedy, or top-k temperature sampling when
  // `sampling` = {temperature, topK, randomSeed} is given (the logits then go through memory).
  async recordHead(recorder, temps, hiddenRow, sampling, tokenOut = this.tokenOut, tokenIndex = 0) {
    const c = this.config;
    if (sampling && !this.logits) this.logits = acquireBuffer(c.vocab * 4, undefined, 'logits');
    await this.recordNormedLmHead(recorder, temps, hiddenRow, tokenOut, tokenIndex, sampling ? this.logits : null);
    if (sampling) {
      await recordGPUSample(recorder, this.logits, c.vocab, Object.assign({ outputBuffer: tokenOut, outputIndex: tokenIndex }, sampling));
    }
  }

  // Pushes prompt tokens (or their next portion) through the batched path, `chunk` tokens per pass, writing KV rows
  // startPos.. ; returns the token after the last one.
  // Mirrors the reference's prefill (src/inference/pipelines/text/generator.js) on the HIP ops.
  async prefill(tokens, startPos = 0, options = {}) {
    const c = this.config;
    const chunk = Math.max(1, Math.min(options.chunk || 2048, tokens.length));
    if (tokens.length === 0 || startPos + tokens.length > c.maxSeq) {
      throw new Error(`[prefill] ${tokens.length} tokens at ${startPos} do not fit maxSeq=${c.maxSeq}`);
    }
    const recorder = createCommandRecorder('prefill');
    const temps = [];
    const ids = acquireBuffer((chunk + 1) * 4, undefined, 'prefill_ids');
    temps.push(ids);
    let rows = null, T = 0;
    this.remember(startPos, tokens);
    for (let c0 = 0; c0 < tokens.length; c0 += chunk) {
      const part = tokens.slice(c0, c0 + chunk);
      T = part.length;
      const pos = startPos + c0;
      this.advance(pos, T);
      uploadData(ids, new Uint32Array([this.tokenBefore(pos)].concat(Array.from(part))));
      rows = await this.recordPrefillChunk(recorder, temps, ids, part, pos);
    }
    const lastRow = createTensor(bufferWindow(rows.buffer, (T - 1) * rows.rowFloats * 4, rows.rowFloats * 4), 'f32',
      [1, rows.rowFloats], 'last_hidden');
    await this.recordHead(recorder, temps, lastRow, options.sampling || null);
    for (const b of temps) recorder.trackTemporaryBuffer(b);
    recorder.submit();
    const bytes = await readBufferSlice(this.tokenOut, 0, 4);
    return new Uint32Array(bytes)[0];
  }

  // prefill + decode loop: returns the generated token ids.  sampling = {temperature, topK, seed}
  // draws token i with randomSeed seed + i (greedy when absent), as the reference's generator
  // advances its seed per step.
  async generate(promptTokens, maxTokens, sampling = null) {
    const draw = (i) => (sampling ? { temperature: sampling.temperature, topK: sampling.topK, randomSeed: sampling.seed + i } : null);
    const out = [];
    let tok = await this.prefill(promptTokens, 0, { sampling: draw(0) });
    out.push(tok);
    for (let i = 1; i < maxTokens; i++) {
      tok = await this.decodeStep(tok, promptTokens.length + i - 1, { sampling: draw(i) });
      out.push(tok);
    }
    return out;
  }

  // Records the ops of one decode step for the token id in this.ids at position `pos`; the new
  // token id goes to this.tokenOut.  Temporaries are pushed onto `temps`.
  // options.idsBuffer / prevBuffer: the input token id, and the one before it, are read from these device words
  // instead; options.tokenOutBuffer / tokenOutIndex: the new token goes to that word of that buffer instead.
  async recordDecodeStep(recorder, temps, pos, options = {}) {
    const c = this.config;
    if (!(pos >= 0 && pos < c.maxSeq)) {
      // the ops take no cache capacity: a position past the caches would write K/V out of bounds
      throw new Error(`[decodeStep] position ${pos} is outside the KV cache (maxSeq=${c.maxSeq})`);
    }
    // a captured step (its key count on the device) is recorded here and runs when it is replayed
    if (!options.deviceKvLen) this.advance(pos, 1);
    const tokenOut = options.tokenOutBuffer || this.tokenOut, tokenIndex = options.tokenOutIndex || 0;
    let x = await this.recordEmbedding(recorder, temps, options.idsBuffer || this.ids, options.prevBuffer || bufferWindow(this.ids, 8, 4),
      pos, options);
    x = await this.recordLayers(recorder, temps, x, pos, options);
    if (options.sampling) {
      await this.recordHead(recorder, temps, x, options.sampling, tokenOut, tokenIndex);
    } else {
      await this.recordNormedLmHead(recorder, temps, x, tokenOut, tokenIndex, options.logitsOutput || null);
    }
  }

  // Returns the greedy token for `token` at position `pos` (KV rows 0..pos-1 present).
  // options.recorder: a recorder of the caller's (e.g. a profiling one) instead of a fresh one.
  async decodeStep(token, pos, options = {}) {
    const recorder = options.recorder || createCommandRecorder('decode');
    const temps = [];
    this.uploadStep(token, pos);
    if (this.finitenessGuard) getNative().fillZero(this.tokenOut.ptr, 4, FINITENESS_STATUS_BYTES);
    await this.recordDecodeStep(recorder, temps, pos, options);
    for (const b of temps) recorder.trackTemporaryBuffer(b);
    recorder.submit();
    // the only device->host crossing: the token, with the guard's status words beside it
    const bytes = await readBufferSlice(this.tokenOut, 0, this.finitenessGuard ? 4 + FINITENESS_STATUS_BYTES : 4);
    const words = new Uint32Array(bytes);
    if (this.finitenessGuard) {
      const status = parseFinitenessStatusWords(words, 1);
      if (status.triggered) throw new FinitenessError(`F16 bounds exceeded during generation${status.metadata}`);
    }
    return words[0];
  }

  // n greedy steps starting with `token` at position `pos`; returns the n new token ids.  Every step's
  // token is read back (4 bytes per step, as in decodeStep), but one step late: step k + 1 takes its input
  // token from device memory and is enqueued before the host waits for token k, whose copy into pinned
  // memory was enqueued behind step k, so the GPU never waits for the host between steps (the reference
  // stages its token readbacks through a ring the same way, src/inference/decode-ring.js:141-177).  A
  // caller with a stop condition checks the tokens as they come and drops the one step in flight.
  async decodeGreedy(token, pos, n) {
    if (n <= 0) return [];
    if (this.finitenessGuard) {
      const guarded = [];
      for (let k = 0; k < n; k++) {
        token = await this.decodeStep(token, pos + k);
        guarded.push(token);
      }
      return guarded;
    }
    const native = getNative();
    if (!this.readback) {
      const host = native.hostAlloc(4 * TOKEN_RING);
      const events = [];
      for (let i = 0; i < READ_EVENTS; i++) events.push(native.eventCreate());
      this.readback = { host, tokens: new Uint32Array(host.view), events, ring: acquireBuffer(4 * TOKEN_RING, undefined, 'token_ring') };
    }
    const rb = this.readback;
    const enqueueStep = async (k) => {
      const recorder = createCommandRecorder('decode');
      const temps = [];
      const slot = k % TOKEN_RING;
      const options = { tokenOutBuffer: rb.ring, tokenOutIndex: slot };
      if (k > 0) {
        options.idsBuffer = bufferWindow(rb.ring, 4 * ((k - 1) % TOKEN_RING), 4);
        options.prevBuffer = k > 1 ? bufferWindow(rb.ring, 4 * ((k - 2) % TOKEN_RING), 4) : bufferWindow(this.ids, 0, 4);
      }
      await this.recordDecodeStep(recorder, temps, pos + k, options);
      for (const b of temps) recorder.trackTemporaryBuffer(b);
      recorder.submit();
      native.downloadAsync(rb.host.ptr, 4 * slot, rb.ring.ptr, 4 * slot, 4);
      native.eventRecord(rb.events[k % READ_EVENTS]);
    };
    const waitToken = (k) => {
      native.eventSynchronize(rb.events[k % READ_EVENTS]);
      return rb.tokens[k % TOKEN_RING];
    };
    this.uploadStep(token, pos);
    await enqueueStep(0);
    const out = [];
    for (let k = 1; k < n; k++) {
      await enqueueStep(k);
      out.push(waitToken(k - 1));
    }
    out.push(waitToken(n - 1));
    this.remember(pos + 1, out);
    return out;
  }

  // Frees the pinned staging memory, the device ring and the events decodeGreedy made.
  releaseReadback() {
    if (this.readback) {
      const native = getNative();
      native.sync();
      for (const ev of this.readback.events) native.eventDestroy(ev);
      this.readback.tokens = null;
      native.hostFree(this.readback.host.ptr);
      releaseBuffer(this.readback.ring);
      this.readback = null;
    }
  }

  // Captures the decode step into a HIP graph, the counterpart of the reference's
  // one-submit-per-step recorder (generator-steps.js:605,814).  The step runs once normally first
  // (every kernel's one-time set-up then lies outside the capture); the buffers the captured step
  // uses stay allocated for the graph's life.
  async captureDecodeStep(token, pos) {
    if (!this.deviceKvLenServed()) throw new Error('[captureDecodeStep] serves the fused-attention step');
    const c = this.config;
    const first = await this.decodeStep(token, pos);
    this.uploadStep(token, pos, pos + 1);
    getNative().graphBegin();
    let graph = null;
    const temps = [];
    try {
      // with the guard on the captured step also clears the status words (the library moves the
      // checks' step number with the position at every replay)
      if (this.finitenessGuard) getNative().fillZero(this.tokenOut.ptr, 4, FINITENESS_STATUS_BYTES);
      await this.recordDecodeStep(createCommandRecorder('decode_capture'), temps, pos, { deviceKvLen: true });
    } finally {
      graph = getNative().graphEnd(pos);
    }
    getNative().graphSetMaxPosition(graph, c.maxSeq - 1);
    this.graph = graph;
    this.graphBuffers = temps;
    return first;
  }

  // One decode step by replaying the captured graph at position `pos`.
  async decodeStepGraph(token, pos) {
    const c = this.config;
    if (!(pos >= 0 && pos < c.maxSeq)) {
      throw new Error(`[decodeStepGraph] position ${pos} is outside the KV cache (maxSeq=${c.maxSeq})`);
    }
    if (!this.graph) return this.captureDecodeStep(token, pos);
    this.advance(pos, 1);
    // token id and key count travel together; the attention kernels of the captured step read the count
    this.uploadStep(token, pos, pos + 1);
    getNative().graphLaunch(this.graph, pos);
    const bytes = await readBufferSlice(this.tokenOut, 0, this.finitenessGuard ? 4 + FINITENESS_STATUS_BYTES : 4);
    const words = new Uint32Array(bytes);
    if (this.finitenessGuard) {
      const status = parseFinitenessStatusWords(words, 1);
      if (status.triggered) throw new FinitenessError(`F16 bounds exceeded during generation${status.metadata}`);
    }
    return words[0];
  }

  releaseGraph() {
    if (this.graph) {
      getNative().graphDestroy(this.graph);
      for (const b of this.graphBuffers) releaseBuffer(b);
      this.graph = null;
      this.graphBuffers = [];
    }
  }

  destroy() {
    this.releaseGraph();
    this.releaseReadback();
    this.releaseWeights();
  }
}
