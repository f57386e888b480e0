// Arguments of the attention kernels (plain and MFMA); mirrored by a ctypes.Structure.
#pragma once

#include "common.h"

struct AttnArgs {
  const void* q;        // [tokens][ldq]; head j at columns j * head_dim
  int64_t ldq;
  void* out;            // [tokens][ldo]
  int64_t ldo;
  const int* tok_seq;   // [tokens]
  const int* tok_pos;   // [tokens]
  const int* seq_off;   // [n_seqs + 1] first token of each sequence in the step
  const int* seq_start; // [n_seqs] position of that first token
  KvView kv;
  int q_heads;
  int n_tokens;
  int n_seqs;
  int max_count;        // most tokens any sequence brings in this step
  int window;           // 0 = all earlier keys
  float scale;
  // With splits > 1 the keys are cut into that many runs, each run is a work-group of its own that
  // leaves (output row, maximum, sum) in `partial` [rows][q_heads][splits][head_dim + 2], and a
  // second kernel joins them into `out`.  Decode: the runs of every sequence's keys, a row is a
  // sequence.  Prompts (bfloat16, heads of 64 to 128, no window): the runs of every query tile's keys, a
  // row is a token of the step.
  int splits;
  float* partial;
  // Decode (bfloat16 MFMA kernels) only: 0, or `out` is chunk-major with that many rows
  // (activation_offset in common.h); ldo is then not used.
  int out_rows;
  // 0, or keys are seen in chunks of that many positions, counted from position 0 of the sequence:
  // a query at position p sees the keys from p - p % chunk through p (and, with a window as well,
  // only those the window also holds).
  int chunk;
  // null, or one logit per query head that stands in every softmax's denominator beside the keys a
  // query sees: exp(sink[head]) is added once, unscaled, with no key and no value of its own (the
  // weights of a query's keys then add up to less than one).
  const float* sink;
  // How a score s = q . k * scale weighs its key.
  //   0: softmax(s) over the keys a query sees
  //   1: softmax(cap * tanh(s / cap))
  //   2: sigmoid(s + score_bias[head]), every key by itself: nothing is normalised over the keys (no sink)
  int form;
  float cap;                // form 1: positive
  const float* score_bias;  // form 2: [q_heads], or null for zero
  // What happens to a head's output row before it is stored: times sigmoid(gate), one float32 logit per head
  // (`gate_span` 0: column `head` of the token's row) or per channel (1: column head * gate_dim + channel; channels
  // from gate_dim on hold zeros and have none); null: no factor.  `out_f32`: stored in 32-bit whatever the products'
  // type.  Forms 1 and 2 and these are in the kernels built with BT_ATTENTION_FORM and in the plain kernel.
  const float* gate;        // [tokens][ld_gate]
  int64_t ld_gate;
  int gate_span;
  int gate_dim;
  int out_f32;
  // The first `keep` positions of a sequence are seen by every later query of it, whatever window and chunk say.
  int keep;
  // attention_shared.hip only: the value channels from here on are zero (0: none is).
  int value_dim;
};

// What a sink adds to a softmax's denominator that is kept relative to the maximum `top`.  The plain and
// the float32 decode kernels keep maxima as natural logarithms, the MFMA kernels in powers of two.
__device__ __forceinline__ float bt_sink_term(const float* sink, int head, float top) {
  return sink ? expf(sink[head] - top) : 0.f;
}
__device__ __forceinline__ float bt_sink_term_pow2(const float* sink, int head, float top) {
  return sink ? exp2f(sink[head] * 1.4426950408889634f - top) : 0.f;
}

__device__ __forceinline__ float bt_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// The gate's factor on channel `channel` of head `head` of token `tok`.
__device__ __forceinline__ float bt_output_gate(const AttnArgs& a, int64_t tok, int head, int channel) {
  if (!a.gate) return 1.f;
  const bool none = a.gate_span == 1 && channel >= a.gate_dim;
  const int column = a.gate_span == 1 ? head * a.gate_dim + (none ? 0 : channel) : head;
  const float factor = bt_sigmoid(a.gate[tok * a.ld_gate + column]);
  return none ? 1.f : factor;
}

// What forms and output stages need of their arguments; nullptr, or what is wrong.
inline const char* bt_check_form(const AttnArgs& a) {
  if (a.form < 0 || a.form > 2) return "unknown form of the scores";
  if (a.form == 1 && !(a.cap > 0.f)) return "the scores' cap must be positive";
  if (a.form == 2 && a.sink) return "a sink stands in a softmax's denominator; sigmoid weights have none";
  if (a.form != 2 && a.score_bias) return "a bias on the scores goes with sigmoid weights";
  if (a.gate && (a.gate_span < 0 || a.gate_span > 1 ||
                 a.ld_gate < (a.gate_span == 1 ? (int64_t)a.q_heads * a.gate_dim : (int64_t)a.q_heads) ||
                 (a.gate_span == 1 && (a.gate_dim <= 0 || a.gate_dim > a.kv.head_dim))))
    return "the gate's rows do not hold a logit per head or channel";
  return nullptr;
}

// The first position a query at `pos` sees: the later of its window's and its chunk's first key (kept first
// positions aside).  It never decreases as `pos` grows, so the first query of a run of queries has the lowest.
__host__ __device__ __forceinline__ int bt_first_seen(int pos, int window, int chunk) {
  int lo = 0;
  if (window > 0 && pos - window + 1 > lo) lo = pos - window + 1;
  if (chunk > 0 && pos - pos % chunk > lo) lo = pos - pos % chunk;
  return lo;
}

// The positions that queries whose first key is `from` or later walk, as one range 0 .. without a gap: the kept first
// positions (in whole tiles), then everything from `from` on.  With nothing kept the range starts at `from`.
struct KeyWalk {
  int kept, skip;
  // the position at place v of the range
  __device__ __forceinline__ int at(int v) const { return v < kept ? v : v + skip; }
  // the place that stands for position `end` (one past the last key, beyond `from`)
  __device__ __forceinline__ int places(int end) const { return end - skip; }
};
// `from` is a multiple of `tile` (a power of two).
__device__ __forceinline__ KeyWalk bt_key_walk(int from, int keep, int tile) {
  KeyWalk walk;
  const int whole = (keep + tile - 1) & ~(tile - 1);
  walk.kept = whole < from ? whole : from;
  walk.skip = from - walk.kept;
  return walk;
}

// Which keys a query sees, for a test of two comparisons: those from `lo` through its own position, and those below `kept`.
struct SeenKeys {
  int lo, kept;
  unsigned span;
  __device__ __forceinline__ bool operator()(int key) const { return (unsigned)(key - lo) <= span || key < kept; }
};
// A column without a query (pos < 0) sees nothing.
__device__ __forceinline__ SeenKeys bt_seen_keys(int pos, int first_seen, int keep) {
  SeenKeys seen;
  seen.lo = pos < 0 ? 1 << 30 : first_seen;
  seen.span = (unsigned)(pos - seen.lo);
  seen.kept = keep < pos + 1 ? keep : pos + 1;
  return seen;
}
