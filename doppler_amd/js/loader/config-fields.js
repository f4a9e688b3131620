// Reading of a design's config.json: fields that must be there, fields that may, and nothing else.
export function configFields(design) {
  function take(obj, where, required, optional = []) {
    if (obj === null || typeof obj !== 'object' || Array.isArray(obj)) throw new Error(`[${design}] ${where} must be an object`);
    const unknown = Object.keys(obj).filter((k) => !required.includes(k) && !optional.includes(k));
    if (unknown.length) throw new Error(`[${design}] ${where} has keys this design does not have: ${unknown}`);
    const missing = required.filter((k) => !(k in obj));
    if (missing.length) throw new Error(`[${design}] ${where} lacks ${missing}`);
    return obj;
  }

  function count(obj, key, where) {
    if (!Number.isInteger(obj[key]) || obj[key] < 1) throw new Error(`[${design}] ${where}.${key} must be a positive integer, got ${obj[key]}`);
    return obj[key];
  }

  function number(obj, key, where, positive = false) {
    if (typeof obj[key] !== 'number' || (positive && !(obj[key] > 0))) {
      throw new Error(`[${design}] ${where}.${key} must be a ${positive ? 'positive ' : ''}number, got ${obj[key]}`);
    }
    return obj[key];
  }

  return { take, count, number };
}
