// Tensors of a safetensors file, checked against the shape the configuration implies.
import fs from 'fs';

export class SafetensorsFile {
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
