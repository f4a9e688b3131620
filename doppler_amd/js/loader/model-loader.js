// Model registry of the JavaScript host: a folder with manifest.json (RDRR, Q4_K) or with config.json +
// model.safetensors, whose `architecture` names a design -> a ready decoder.
import fs from 'fs';
import path from 'path';

import { loadDecoderWeights } from './rdrr-loader.js';
import { loadGusolorn } from './gusolorn-loader.js';
import { loadZepavik } from './zepavik-loader.js';
import { HipTextDecoder } from '../pipeline/decode-step.js';
import { DenseTextDecoder } from '../pipeline/dense-decoder.js';

const dense = (load) => (dir, options) => {
  const { config, weights } = load(dir, options.maxSeq);
  return new DenseTextDecoder(Object.assign({ compute: options.dtype === 'float32' ? 'f32' : 'bf16' }, config, options.config), weights);
};
const ARCHITECTURES = { Zepavik: dense(loadZepavik), Gusolorn: dense(loadGusolorn) };

// options: {maxSeq, dtype: 'bfloat16'|'float32', config: extra decoder settings}
export function loadModel(dir, options = {}) {
  if (fs.existsSync(path.join(dir, 'manifest.json'))) {
    if (options.dtype === 'float32') throw new Error('[loadModel] RDRR Q4_K models do not run in float32');
    const { config, weights } = loadDecoderWeights(dir, options.maxSeq || 4096);
    return new HipTextDecoder(Object.assign({}, config, options.config), weights);
  }
  const file = path.join(dir, 'config.json');
  if (!fs.existsSync(file)) throw new Error(`[loadModel] ${dir} holds neither manifest.json nor config.json`);
  const name = JSON.parse(fs.readFileSync(file, 'utf8')).architecture;
  if (!Object.prototype.hasOwnProperty.call(ARCHITECTURES, name)) throw new Error(`[loadModel] architecture "${name}" is not one of ${Object.keys(ARCHITECTURES)}`);
  return ARCHITECTURES[name](dir, options);
}
