// Gusolorn models (config.json + model.safetensors) -> {config, weights} of DenseTextDecoder: the JavaScript side of
// doppler_amd/gusolorn.py.  Unknown configuration keys fail closed with their names.
import fs from 'fs';
import path from 'path';

import { configFields } from './config-fields.js';
import { SafetensorsFile } from './safetensors-file.js';

const DEFAULT_POSITIONS = 4096;
const { take, count, number } = configFields('gusolorn');
const given = (x) => x !== null && x !== undefined;

function latent(m, at, i, entries) {
  take(m, at, ['heads', 'dim', 'rot_dim', 'vdim', 'kv_rank', 'scale', 'rot'], ['mask', 'kv_from']);
  const rot = take(m.rot, `${at}.rot`, ['base', 'dims']);
  const rotDim = count(m, 'rot_dim', at);
  if (rotDim % 2 || rot.dims !== rotDim) throw new Error(`[gusolorn] ${at}: the rotated part of ${rotDim} elements must be even and rotated whole`);
  if (given(m.kv_from)) {
    const lender = Number.isInteger(m.kv_from) && m.kv_from >= 0 && m.kv_from < i ? entries[m.kv_from] : null;
    if (!lender || lender.type !== 'latent_attention' || given(lender.mixer.kv_from)) {
      throw new Error(`[gusolorn] ${at}.kv_from ${m.kv_from} is not an earlier layer with latent rows of its own`);
    }
    const o = lender.mixer;
    if (o.kv_rank !== m.kv_rank || o.rot_dim !== m.rot_dim || o.rot.base !== rot.base || o.rot.dims !== rot.dims) {
      throw new Error(`[gusolorn] ${at}.kv_from: kv_rank, rot_dim and rot must be those of layer ${m.kv_from}`);
    }
  }
  return {
    type: 'latent_attention', heads: count(m, 'heads', at), dim: count(m, 'dim', at), rotDim, vdim: count(m, 'vdim', at),
    kvRank: count(m, 'kv_rank', at), scale: number(m, 'scale', at), rotBase: number(rot, 'base', `${at}.rot`, true),
    window: given(m.mask) ? count(take(m.mask, `${at}.mask`, ['size']), 'size', `${at}.mask`) : 0, kvFrom: given(m.kv_from) ? m.kv_from : null,
  };
}

function memory(m, at) {
  take(m, at, ['heads', 'dim', 'vdim', 'gate_cap']);
  return { type: 'mlstm', heads: count(m, 'heads', at), dim: count(m, 'dim', at), vdim: count(m, 'vdim', at), gateCap: number(m, 'gate_cap', at, true) };
}

function feedForward(mlp, at) {
  if (!given(mlp)) return null;
  if (mlp.kind === 'dense') return { type: 'dense', ff: count(take(mlp, at, ['kind', 'ff']), 'ff', at), activation: 'gelu_erf' };
  if (mlp.kind !== 'moe') throw new Error(`[gusolorn] ${at}.kind "${mlp.kind}" is not a feed-forward of this design`);
  take(mlp, at, ['kind', 'router', 'expert'], ['shared']);
  take(mlp.router, `${at}.router`, ['experts', 'top']);
  const width = (e, w) => ({ ff: count(take(e, w, ['ff', 'limit']), 'ff', w), limit: number(e, 'limit', w) });
  const experts = count(mlp.router, 'experts', `${at}.router`), top = count(mlp.router, 'top', `${at}.router`);
  if (top > experts) throw new Error(`[gusolorn] ${at}.router.top ${top} exceeds ${experts} experts`);
  return Object.assign({ type: 'experts', experts, top, shared: given(mlp.shared) ? width(mlp.shared, `${at}.shared`) : null },
    width(mlp.expert, `${at}.expert`));
}

const MIXERS = { latent_attention: latent, mlstm: memory };

export function gusolornConfig(c) {
  take(c, 'config', ['architecture', 'layers', 'norm', 'vocab', 'width']);
  const layers = c.layers.map((entry, i) => {
    const where = `layers[${i}]`;
    take(entry, where, ['type', 'mixer'], ['mlp']);
    if (!Object.prototype.hasOwnProperty.call(MIXERS, entry.type)) throw new Error(`[gusolorn] ${where}.type "${entry.type}" is not a mixer of this design`);
    return { sequential: true, mixer: MIXERS[entry.type](entry.mixer, `${where}.mixer`, i, c.layers), mlp: feedForward(entry.mlp, `${where}.mlp`) };
  });
  return {
    hidden: count(c, 'width', 'config'), vocab: count(c, 'vocab', 'config'), eps: number(take(c.norm, 'norm', ['eps']), 'eps', 'norm'), logitScale: 1,
    maxPositions: 0, bigram: null, layers,
  };
}

export function loadGusolorn(dir, maxSeq) {
  const config = gusolornConfig(JSON.parse(fs.readFileSync(path.join(dir, 'config.json'), 'utf8')));
  config.maxSeq = maxSeq || DEFAULT_POSITIONS;
  const file = new SafetensorsFile(path.join(dir, 'model.safetensors')), W = config.hidden, V = config.vocab;
  const aroundZero = (name, shape) => file.f32(name, shape).map((x) => 1 + x);

  function mixer(m, p) {
    const H = m.heads, d = m.dim, e = m.vdim;
    if (m.type === 'mlstm') {
      return {
        q: file.bf16(`${p}q`, [H * d, W]), k: file.bf16(`${p}k`, [H * d, W]), v: file.bf16(`${p}v`, [H * e, W]), g: file.bf16(`${p}g`, [H * e, W]),
        i: file.bf16(`${p}i`, [H, W]), f: file.bf16(`${p}f`, [H, W]), iBias: file.f32(`${p}i.b`, [H]), fBias: file.f32(`${p}f.b`, [H]),
        headNorm: file.f32(`${p}norm`, [H * e]), o: file.bf16(`${p}o`, [W, H * e]),
      };
    }
    const w = {
      q: file.bf16(`${p}q`, [H * (d + m.rotDim), W]), uk: file.bf16(`${p}uk`, [H * d, m.kvRank]), uv: file.bf16(`${p}uv`, [H * e, m.kvRank]),
      o: file.bf16(`${p}o`, [W, H * e]),
    };
    if (m.kvFrom === null) {
      w.dkv = file.bf16(`${p}dkv`, [m.kvRank + m.rotDim, W]);
      w.latentNorm = file.f32(`${p}dkv.norm`, [m.kvRank]);
    }
    return w;
  }

  function feedForwardWeights(mlp, p) {
    if (mlp.type === 'dense') return { up: file.bf16(`${p}up`, [mlp.ff, W]), down: file.bf16(`${p}down`, [W, mlp.ff]) };
    const each = (name, shape) => Array.from({ length: mlp.experts }, (_, k) => file.bf16(`${p}e${k}.${name}`, shape));
    const w = { router: file.bf16(`${p}router`, [mlp.experts, W]), gate: each('gate', [mlp.ff, W]), up: each('up', [mlp.ff, W]), down: each('down', [W, mlp.ff]) };
    if (mlp.shared) {
      const s = mlp.shared.ff;
      Object.assign(w, {
        sharedGate: file.bf16(`${p}shared.gate`, [s, W]), sharedUp: file.bf16(`${p}shared.up`, [s, W]), sharedDown: file.bf16(`${p}shared.down`, [W, s]),
        sharedSg: file.bf16(`${p}shared.sg`, [1, W]),
      });
    }
    return w;
  }

  try {
    const layers = config.layers.map((l, i) => {
      const w = { norm1: aroundZero(`l${i}.norm1`, [W]), ls1: file.f32(`l${i}.ls1`, [W]), mixer: mixer(l.mixer, `l${i}.mix.`) };
      if (l.mlp) {
        Object.assign(w, { norm2: aroundZero(`l${i}.norm2`, [W]), ls2: file.f32(`l${i}.ls2`, [W]), mlp: feedForwardWeights(l.mlp, `l${i}.mlp.`) });
      }
      return w;
    });
    return { config, weights: { embed: file.bf16('embed', [V, W]), head: file.bf16('head', [V, W]), finalNorm: aroundZero('final.norm', [W]), layers } };
  } finally {
    file.close();
  }
}
