// Driver of the tests of the JavaScript host with whole models: node run_models.mjs jobs.json -> one JSON line with the tokens of every job.
import fs from 'fs';
import { loadModel } from '../../doppler_amd/js/loader/model-loader.js';

async function main() {
  const jobs = JSON.parse(fs.readFileSync(process.argv[2], 'utf8'));
  const results = {};
  for (const j of jobs) {
    const dec = loadModel(j.dir, { maxSeq: j.maxSeq, dtype: j.dtype, config: j.config });
    const n = j.prompt.length;
    let tokens;
    if (j.mode === 'generate') {
      tokens = await dec.generate(j.prompt, j.count, j.sampling || null);
    } else if (j.mode === 'portions') {
      let tok = null, at = 0;
      for (const size of j.sizes) {
        tok = size === 1 ? await dec.decodeStep(j.prompt[at], at) : await dec.prefill(j.prompt.slice(at, at + size), at, { chunk: j.chunk });
        at += size;
      }
      tokens = [tok];
      for (let i = 1; i < j.count; i++) tokens.push(await dec.decodeStep(tokens[i - 1], n + i - 1));
    } else if (j.mode === 'greedy') {
      const first = await dec.prefill(j.prompt);
      tokens = [first].concat(await dec.decodeGreedy(first, n, j.count - 1));
      // again over the same positions: the pinned ring and the cache rows are reused
      const second = await dec.prefill(j.prompt);
      const again = [second].concat(await dec.decodeGreedy(second, n, j.count - 1));
      if (JSON.stringify(again) !== JSON.stringify(tokens)) throw new Error(`decodeGreedy repeated differently: ${again}`);
    } else if (j.mode === 'graph') {
      tokens = [await dec.prefill(j.prompt)];
      for (let i = 1; i < j.count; i++) {
        const pos = n + i - 1;
        tokens.push(i % 5 === 4 ? await dec.decodeStep(tokens[i - 1], pos) : await dec.decodeStepGraph(tokens[i - 1], pos));
      }
    } else if (j.mode === 'order') {
      tokens = [];
      await dec.prefill(j.prompt);
      for (const run of [() => dec.decodeStep(1, n + 2), () => dec.prefill([1, 2], n - 1), () => dec.decodeStep(1, n)]) {
        try { await run(); tokens.push('ran'); } catch (e) { tokens.push(e.message); }
      }
    } else if (j.mode === 'guard') {
      let message = 'did not throw';
      const first = await dec.prefill(j.prompt);
      try { await dec.decodeStep(first, n); } catch (e) { message = `${e.name}: ${e.message}`; }
      tokens = [message];
    }
    dec.destroy();
    results[j.name] = tokens;
  }
  console.log(JSON.stringify(results));
}

main().catch((e) => { console.error(e.stack || String(e)); process.exit(1); });
