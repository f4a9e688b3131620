// Zepavik models (config.json + model.safetensors) -> {config, weights} of DenseTextDecoder.  Unknown configuration keys
// fail closed with their names.
import fs from 'fs';
import path from 'path';

function take(obj, where, required, optional = []) {
  if (obj === null || typeof obj !== 'object' || Array.isArray(obj)) throw new Error(`[zepavik] ${where} must be an object`);
  const unknown = Object.keys(obj).filter((k) => !required.includes(k) && !optional.includes(k));
  if (unknown.length) throw new Error(`[zepavik] ${where} has keys this design does not have: ${unknown}`);
  const missing = required.filter((k) => !(k in obj));
  if (missing.length) throw new Error(`[zepavik] ${where} lacks ${missing}`);
  return obj;
}

function count(obj, key, where) {
  if (!Number.isInteger(obj[key]) || obj[key] < 1) throw new Error(`[zepavik] ${where}.${key} must be a positive integer, got ${obj[key]}`);
  return obj[key];
}

export function zepavikConfig(c) {
  take(c, 'config', ['architecture', 'embedding', 'layers', 'logit_scale', 'max_positions', 'norm', 'vocab', 'width']);
  const b = take(take(c.embedding, 'embedding', ['bigram']).bigram, 'embedding.bigram', ['buckets', 'mul_prev', 'mul_cur']);
  const layers = c.layers.map((entry, i) => {
    const where = `layers[${i}]`;
    take(entry, where, ['type', 'mixer'], ['mlp']);
    if (entry.type !== 'attention') throw new Error(`[zepavik] ${where}.type "${entry.type}" is not a mixer of this design`);
    const m = take(entry.mixer, `${where}.mixer`, ['heads', 'kv_heads', 'dim', 'vdim', 'scale', 'mask']);
    const mask = take(m.mask, `${where}.mixer.mask`, ['size']);
    const heads = count(m, 'heads', where), kvHeads = count(m, 'kv_heads', where);
    if (heads % kvHeads) throw new Error(`[zepavik] ${where}: ${heads} heads are not a multiple of ${kvHeads} key/value heads`);
    let mlp = null;
    if (entry.mlp !== null && entry.mlp !== undefined) {
      take(entry.mlp, `${where}.mlp`, ['kind', 'ff']);
      if (entry.mlp.kind !== 'dense') throw new Error(`[zepavik] ${where}.mlp.kind "${entry.mlp.kind}" is not a feed-forward of this design`);
      mlp = { ff: count(entry.mlp, 'ff', where), activation: 'relu2' };
    }
    return {
      mixer: { heads, kvHeads, dim: count(m, 'dim', where), vdim: count(m, 'vdim', where), window: count(mask, 'size', where), scale: m.scale,
        logBias: true, valueNorm: true, gate: true },
      mlp,
    };
  });
  return {
    hidden: count(c, 'width', 'config'), vocab: count(c, 'vocab', 'config'), eps: take(c.norm, 'norm', ['eps']).eps, logitScale: c.logit_scale,
    maxPositions: count(c, 'max_positions', 'config'),
    bigram: { buckets: count(b, 'buckets', 'embedding.bigram'), mulPrev: b.mul_prev, mulCur: b.mul_cur }, layers,
  };
}

class SafetensorsFile {
  constructor(file) {
    this.fd = fs.openSync(file, 'r');
    const len = Buffer.alloc(8);
    fs.readSync(this.fd, len, 0, 8, 0);
    const n = Number(len.readBigUInt64LE(0));
    const text = Buffer.alloc(n);
    fs.readSync(this.fd, text, 0, n, 8);
    this.header = JSON.parse(text.toString('utf8'));
    this.base = 8 + n;
  }

  bf16(name, shape) {
    const t = this.header[name];
    if (!t) throw new Error(`Tensor '${name}' is not in the file`);
    if (t.dtype !== 'BF16' || t.shape.length !== shape.length || t.shape.some((x, i) => x !== shape[i])) {
      throw new Error(`Tensor '${name}' is ${t.dtype} [${t.shape}], the configuration implies BF16 [${shape}]`);
    }
    const elements = shape.reduce((a, x) => a * x, 1), [a, b] = t.data_offsets;
    if (b - a !== 2 * elements) throw new Error(`Tensor '${name}' does not fit its data range`);
    const out = new Uint16Array(elements);
    const bytes = new Uint8Array(out.buffer);
    for (let at = 0; at < bytes.length;) {
      const got = fs.readSync(this.fd, bytes, at, Math.min(bytes.length - at, 1 << 28), this.base + a + at);
      if (got <= 0) throw new Error(`Tensor '${name}' reaches past the end of the file`);
      at += got;
    }
    return out;
  }

  f32(name, shape) {
    const bits = this.bf16(name, shape), wide = new Uint32Array(bits.length);
    for (let i = 0; i < bits.length; i++) wide[i] = bits[i] << 16;
    return new Float32Array(wide.buffer);
  }

  close() {
    fs.closeSync(this.fd);
  }
}

export function loadZepavik(dir, maxSeq) {
  const config = zepavikConfig(JSON.parse(fs.readFileSync(path.join(dir, 'config.json'), 'utf8')));
  config.maxSeq = maxSeq ? Math.min(maxSeq, config.maxPositions) : config.maxPositions;
  const file = new SafetensorsFile(path.join(dir, 'model.safetensors')), W = config.hidden, V = config.vocab;
  try {
    const layers = config.layers.map(({ mixer: m, mlp }, i) => {
      const p = `l${i}.mix.`, H = m.heads, G = m.kvHeads;
      const w = {
        norm: file.f32(`l${i}.norm1`, [W]), q: file.bf16(`${p}q`, [H * m.dim, W]), qBias: file.f32(`${p}q.b`, [H * m.dim]),
        k: file.bf16(`${p}k`, [G * m.dim, W]), kBias: file.f32(`${p}k.b`, [G * m.dim]), v: file.bf16(`${p}v`, [G * m.vdim, W]),
        vBias: file.f32(`${p}v.b`, [G * m.vdim]), biasR1: file.f32(`${p}r1`, [H]), biasR2: file.f32(`${p}r2`, [H]),
        gate: file.bf16(`${p}g`, [H, W]), o: file.bf16(`${p}o`, [W, H * m.vdim]),
      };
      if (mlp) {
        w.up = file.bf16(`l${i}.mlp.up`, [mlp.ff, W]);
        w.down = file.bf16(`l${i}.mlp.down`, [W, mlp.ff]);
      }
      return w;
    });
    const weights = {
      embed: file.bf16('embed', [V, W]), bigram: file.bf16('bigram', [config.bigram.buckets + 1, W]),
      pos: file.bf16('pos', [config.maxPositions, W]), head: file.bf16('head', [V, W]), finalNorm: file.f32('final.norm', [W]), layers,
    };
    return { config, weights };
  } finally {
    file.close();
  }
}
