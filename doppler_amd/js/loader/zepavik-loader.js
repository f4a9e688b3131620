// Zepavik models (config.json + model.safetensors) -> {config, weights} of DenseTextDecoder.  Unknown configuration keys
// fail closed with their names.
import fs from 'fs';
import path from 'path';

import { configFields } from './config-fields.js';
import { SafetensorsFile } from './safetensors-file.js';

const { take, count } = configFields('zepavik');

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
