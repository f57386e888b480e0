// bfloat16 attention for heads wider than 128 whose queries all share ONE cached head (attention on a latent: kv_heads is
// one, keys and values lie in the cache at up to 768 channels), and for more query heads on one cached head than the
// ordinary decode kernel takes.  Prompts and decode steps.
//
// A row is one (token, query head) pair; a sequence's rows lie one behind the other, token by token, and since all of them
// meet the same cached vectors a work-group takes 16, 32 or 64 of them whatever tokens they belong to.  Its eight waves divide
// every block of 64 keys between them so that each cached byte is read once a work-group, straight into the registers it
// is multiplied from:
//   scores   wave w multiplies 16 of the keys (w % 4) by one half of the channels (w / 4); the two halves' sums meet in LDS.
//   softmax  two waves for every 16 rows, each with half of the keys (both work out the running maximum over all 64); the
//            probabilities go through LDS in the order of the next product's operand, with the factor the running sums of
//            their row are to be multiplied with.
//   values   wave w owns the blocks of 16 output channels w, w + 8, ...: it reads those channels' values of the block and
//            adds to its own sums, which no other wave touches.
// Two barriers a block.  The values of a block are asked for before its scores are multiplied and the keys of the next
// one right after, so that both are on their way during the softmax.  Both products are v_mfma_f32_16x16x32_bf16 with the
// operands laid out as in attention_bf16.hip (keys and values as "A", rows as "B"), maxima in powers of two, 32-bit sums.
// Channels of the value from `value_dim` on are zero in the cache and are neither read nor multiplied.
//
// With splits > 1 the blocks a tile of rows walks are cut into that many runs, a work-group each, whose results
// attention_shared_join_kernel joins: a decode step has few tiles, and so has a short portion of a prompt.

#include "host.h"
#include "attention.h"
#include "calls.h"

#define SHARED_WAVES 8
#define SHARED_MANY 128       // work-groups of 64 rows from which on they are that large
#define LOG2_E 1.4426950408889634f

__device__ __forceinline__ bf16x8 load_bf16x8(const bf16_t* p) { return *reinterpret_cast<const bf16x8*>(p); }

// A barrier that waits for LDS only: loads from memory stay in flight across it.
__device__ __forceinline__ void lds_barrier() {
  asm volatile("" ::: "memory");
  __builtin_amdgcn_s_waitcnt(0xC07F);                      // lgkmcnt(0)
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}

// HS: steps of 32 channels in half of a head; NV: blocks of 16 value channels a wave owns; NQ: blocks of 16 rows.  The time of
// a block is the time its keys and values take to arrive, so the more rows share them the better: four blocks of rows keep
// their queries in LDS (QUERIES_IN_LDS), in the order of the operand, where the registers do not hold them.
template <int HS, int NV, int NQ>
__global__ void __launch_bounds__(SHARED_WAVES * 64)
attention_shared_kernel(AttnArgs a, int tiles_max) {
  constexpr bool QUERIES_IN_LDS = NQ > 2;
  constexpr int QREG = QUERIES_IN_LDS ? 1 : NQ;
  extern __shared__ bf16x8 s_queries[];                    // QUERIES_IN_LDS: [half of the channels][step][rows][lane]
  __shared__ floatx4 s_scores[2][NQ][4][64];               // [half of the channels][rows][16 keys][lane]
  __shared__ bf16x8 s_probs[NQ][2][64];                    // [rows][half of the keys][lane]
  __shared__ float s_alpha[NQ][16], s_max[NQ][16], s_sum[NQ][2][16];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int i16 = lane & 15, g = lane >> 4;
  const int kt = wave & 3, half = wave >> 2;
  const int HD = a.kv.head_dim, heads = a.q_heads;
  const int vd = a.value_dim > 0 ? a.value_dim : HD;
  const int seq = blockIdx.x % a.n_seqs, tile = tiles_max - 1 - blockIdx.x / a.n_seqs;       // (latest rows first: the longest walks)
  const int off = a.seq_off[seq], count = a.seq_off[seq + 1] - off, start = a.seq_start[seq];
  const int rows = count * heads, row0 = tile * 16 * NQ;
  if (row0 >= rows) return;                                // the whole work-group: this sequence is shorter
  const int last_row = (row0 + 16 * NQ < rows ? row0 + 16 * NQ : rows) - 1;
  const int first_pos = start + row0 / heads, last_pos = start + last_row / heads;
  const int first_seen = bt_first_seen(first_pos, a.window, a.chunk);
  const KeyWalk walk = bt_key_walk(first_seen / BT_KV_BLOCK, (a.keep + BT_KV_BLOCK - 1) / BT_KV_BLOCK, 1);      // (in blocks)
  const int places = walk.places(last_pos / BT_KV_BLOCK) + 1;
  const int splits = a.splits > 1 ? a.splits : 1, split = blockIdx.y;
  const int per_split = (places + splits - 1) / splits;
  const int begin = split * per_split, end = begin + per_split < places ? begin + per_split : places;

  const bf16_t* Q = static_cast<const bf16_t*>(a.q);
  const bf16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  bf16x8 q[QREG][HS];
#pragma unroll
  for (int nq = 0; nq < NQ; ++nq) {
    if (QUERIES_IN_LDS && nq != kt) continue;              // (a wave brings one block of rows for its half of the channels)
    const int r = row0 + 16 * nq + i16, rr = r < rows ? r : rows - 1;
    const bf16_t* row = Q + (int64_t)(off + rr / heads) * a.ldq + rr % heads * HD;
#pragma unroll
    for (int s = 0; s < HS; ++s) {
      const int channel = (half * HS + s) * 32 + g * 8;
      q[QUERIES_IN_LDS ? 0 : nq][s] = channel < HD ? load_bf16x8(row + channel) : zero8;
    }
  }
  bf16x8* my_queries = s_queries + half * HS * NQ * 64 + lane;
  if constexpr (QUERIES_IN_LDS) {
    static_assert(NQ == 4, "four waves, four blocks of rows");
#pragma unroll
    for (int s = 0; s < HS; ++s) my_queries[(s * NQ + kt) * 64] = q[0][s];
    lds_barrier();
  }
  // what this wave does in the softmax: rows 16 * sq + i16, keys 32 * sh .. + 31 of a block
  const bool weighs = wave < 2 * NQ;
  const int sq = weighs ? wave >> 1 : 0, sh = wave & 1;
  const int my_row = row0 + 16 * sq + i16;
  const int my_pos = my_row < rows ? start + my_row / heads : -1;
  const SeenKeys seen = bt_seen_keys(my_pos, my_pos < 0 ? 0 : bt_first_seen(my_pos, a.window, a.chunk), a.keep);
  const int last_seen = bt_first_seen(last_pos, a.window, a.chunk);        // the first position that every row sees
  const float c = a.scale * LOG2_E;
  float m = -INFINITY, l = 0.f;

  floatx4 o[NQ][NV];
#pragma unroll
  for (int nq = 0; nq < NQ; ++nq)
#pragma unroll
    for (int j = 0; j < NV; ++j) o[nq][j] = floatx4{0.f, 0.f, 0.f, 0.f};

  // Addresses: a base that is the same for the whole wave and a 32-bit distance of the lane's, so that few registers hold them.
  const unsigned char* keys = static_cast<const unsigned char*>(a.kv.keys);
  const unsigned char* values = static_cast<const unsigned char*>(a.kv.values);
  const int* block_row = a.kv.blocks + (int64_t)seq * a.kv.max_blocks;
  constexpr int SURE = HS > 4 ? HS - 4 : 0;                // steps that lie inside the head whatever its size is
  const unsigned key_row = (unsigned)(16 * kt + i16) * HD * 2, key_at = key_row + (half * HS * 32 + g * 8) * 2;
  unsigned key_tail[HS - SURE];                            // (a step behind the head reads the row's start and meets zeros of the query)
#pragma unroll
  for (int s = SURE; s < HS; ++s) key_tail[s - SURE] = (half * HS + s) * 32 + g * 8 < HD ? key_at + s * 64 : key_row;
  const unsigned value_at = (unsigned)(g * HD + i16) * 8;
  bf16x8 k[HS];
  bf16x8 v[NV][2];                                         // positions 32 h + 4 g .. + 3 and 32 h + 16 + 4 g .. + 3 of a channel
  auto fetch_keys = [&](int64_t plane) {
    const unsigned char* base = keys + plane * 2;
#pragma unroll
    for (int s = 0; s < HS; ++s)
      k[s] = *reinterpret_cast<const bf16x8*>(base + (s < SURE ? key_at + s * 64 : key_tail[s < SURE ? 0 : s - SURE]));
  };
  int64_t plane = 0, next_plane = 0;
  if (begin < end) {
    plane = kv_plane(a.kv, block_row[walk.at(begin)], 0);
    fetch_keys(plane);
    next_plane = kv_plane(a.kv, block_row[walk.at(begin + 1 < end ? begin + 1 : begin)], 0);
  }
  for (int place = begin; place < end; ++place) {
    const int kb = walk.at(place) * BT_KV_BLOCK;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int dt = SHARED_WAVES * j + wave;
      const unsigned char* base = values + plane * 2 + (16 * dt < vd ? 128 * dt : 0);            // (a block too many reads the first again)
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        const bf16x4 near = *reinterpret_cast<const bf16x4*>(base + (int64_t)64 * HD * h + value_at);
        const bf16x4 far = *reinterpret_cast<const bf16x4*>(base + (int64_t)64 * HD * h + 32 * HD + value_at);
        v[j][h] = __builtin_shufflevector(near, far, 0, 1, 2, 3, 4, 5, 6, 7);
      }
    }
    floatx4 acc[NQ];
#pragma unroll
    for (int nq = 0; nq < NQ; ++nq) acc[nq] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < HS; ++s)
#pragma unroll
      for (int nq = 0; nq < NQ; ++nq) {
        const bf16x8 operand = QUERIES_IN_LDS ? my_queries[(s * NQ + nq) * 64] : q[QUERIES_IN_LDS ? 0 : nq][s];
        acc[nq] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k[s], operand, acc[nq], 0, 0, 0);
      }
#pragma unroll
    for (int nq = 0; nq < NQ; ++nq) s_scores[half][nq][kt][lane] = acc[nq];
    plane = next_plane;
    if (place + 1 < end) {
      fetch_keys(plane);
      next_plane = kv_plane(a.kv, block_row[walk.at(place + 2 < end ? place + 2 : place + 1)], 0);
    }
    lds_barrier();                                         // the scores of the block are in place
    if (weighs) {
      floatx4 x[4];
#pragma unroll
      for (int t = 0; t < 4; ++t) x[t] = s_scores[0][sq][t][lane] + s_scores[1][sq][t][lane];
      const bool whole = kb + BT_KV_BLOCK - 1 <= first_pos && kb >= last_seen;       // (every row sees the whole block)
      if (!whole) {
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
          for (int r = 0; r < 4; ++r) x[t][r] = seen(kb + 16 * t + 4 * g + r) ? x[t][r] : -INFINITY;
      }
      float top = -INFINITY;
#pragma unroll
      for (int t = 0; t < 4; ++t) top = fmaxf(top, fmaxf(fmaxf(x[t][0], x[t][1]), fmaxf(x[t][2], x[t][3])));
      top = fmaxf(top, __shfl_xor(top, 16, 64));
      top = fmaxf(top, __shfl_xor(top, 32, 64));
      const float next = fmaxf(m, top * c);
      const float alpha = next == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(m - next);      // (2^-inf = 0 before the first key seen)
      const float use = next == -INFINITY ? 0.f : next;
      m = next;
      bf16x8 p;
      float sum = 0.f;
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float s = sh ? x[2 + t][r] : x[t][r];
          const float w = __builtin_amdgcn_exp2f(fmaf(s, c, -use));
          sum += w;
          p[4 * t + r] = (bf16_t)w;
        }
      l = fmaf(l, alpha, sum);
      s_probs[sq][sh][lane] = p;
      if (sh == 0 && g == 0) s_alpha[sq][i16] = alpha;
    }
    lds_barrier();                                         // the probabilities of the block are in place
    bf16x8 p[NQ][2];
#pragma unroll
    for (int nq = 0; nq < NQ; ++nq) {
      const float alpha = s_alpha[nq][i16];
      p[nq][0] = s_probs[nq][0][lane];
      p[nq][1] = s_probs[nq][1][lane];
      if (__builtin_amdgcn_ballot_w64(alpha != 1.f) != 0) {
#pragma unroll
        for (int j = 0; j < NV; ++j)
#pragma unroll
          for (int r = 0; r < 4; ++r) o[nq][j][r] *= alpha;
      }
    }
    const int beyond = last_pos + 1 - kb;                  // positions of the block from here on hold no token of any row (0 * NaN is NaN)
#pragma unroll
    for (int j = 0; j < NV; ++j) {
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        bf16x8 w = v[j][h];
        if (beyond < BT_KV_BLOCK) {
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            if (32 * h + 4 * g + r >= beyond) w[r] = (bf16_t)0.f;
            if (32 * h + 16 + 4 * g + r >= beyond) w[4 + r] = (bf16_t)0.f;
          }
        }
#pragma unroll
        for (int nq = 0; nq < NQ; ++nq) o[nq][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w, p[nq][h], o[nq][j], 0, 0, 0);
      }
    }
  }
  if (weighs) {
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (g == 0) {
      s_sum[sq][sh][i16] = l;
      if (sh == 0) s_max[sq][i16] = m;
    }
  }
  lds_barrier();
#pragma unroll
  for (int nq = 0; nq < NQ; ++nq) {
    const int r = row0 + 16 * nq + i16;
    if (r >= rows) continue;
    const int tok = off + r / heads, head = r % heads;
    float total = s_sum[nq][0][i16] + s_sum[nq][1][i16];
    const float top = s_max[nq][i16];
    if (splits > 1) {                                      // this run's share, for attention_shared_join_kernel
      float* record = a.partial + (((int64_t)tok * heads + head) * splits + split) * (HD + 2);
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const int channel = 16 * (SHARED_WAVES * j + wave) + 4 * g;
        typedef __attribute__((__vector_size__(2 * sizeof(float)))) float float2v;
        if (channel < vd) {                                // (value_dim is a multiple of four; records are 8-byte aligned)
          *reinterpret_cast<float2v*>(record + channel) = float2v{o[nq][j][0], o[nq][j][1]};
          *reinterpret_cast<float2v*>(record + channel + 2) = float2v{o[nq][j][2], o[nq][j][3]};
        }
      }
      if (wave == 0 && g == 0) {
        record[HD] = top;
        record[HD + 1] = total;
      }
      continue;
    }
    if (top != -INFINITY) total += bt_sink_term_pow2(a.sink, head, top);
    const float inv = total > 0.f ? 1.0f / total : 0.f;
    const float whole_gate = a.gate && a.gate_span == 0 ? bt_output_gate(a, tok, head, 0) : 1.f;
    bf16_t* out = static_cast<bf16_t*>(a.out);
    for (int dt = wave; 16 * dt < HD; dt += SHARED_WAVES) {
      const int channel = 16 * dt + 4 * g, j = dt / SHARED_WAVES;
      float y[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int jj = 0; jj < NV; ++jj)                      // (no register array is indexed by a variable)
        if (jj == j && channel < vd) {
#pragma unroll
          for (int i = 0; i < 4; ++i)
            y[i] = o[nq][jj][i] * inv * (a.gate && a.gate_span == 1 ? bt_output_gate(a, tok, head, channel + i) : whole_gate);
        }
      bf16x4 packed = {(bf16_t)y[0], (bf16_t)y[1], (bf16_t)y[2], (bf16_t)y[3]};
      *reinterpret_cast<bf16x4*>(out + activation_offset<bf16_t>(a.out_rows, a.ldo, tok, head * HD + channel)) = packed;
    }
  }
}

// Joins the runs: a wave per (token, query head), four to a work-group.  Lane s holds run s's factor; a run that saw no
// key has the maximum -inf and whatever else in its record.
__global__ void __launch_bounds__(256)
attention_shared_join_kernel(AttnArgs a) {
  const int lane = threadIdx.x & 63, HD = a.kv.head_dim, vd = a.value_dim > 0 ? a.value_dim : HD;
  const int64_t pair = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (pair >= (int64_t)a.n_tokens * a.q_heads) return;     // (a whole wave; there is no barrier)
  const int tok = (int)(pair / a.q_heads), head = (int)(pair % a.q_heads);
  const float* runs = a.partial + pair * a.splits * (HD + 2);
  const bool there = lane < a.splits;
  const float* mine = runs + (int64_t)(there ? lane : 0) * (HD + 2);
  const float m = there ? mine[HD] : -INFINITY, l = mine[HD + 1];
  const float top = wave_max(m);
  const float factor = m == -INFINITY ? 0.f : exp2f(m - top);             // (the maxima are kept in powers of two)
  float den = wave_sum(factor > 0.f ? l * factor : 0.f);
  if (top != -INFINITY) den += bt_sink_term_pow2(a.sink, head, top);
  const float inv = den > 0.f ? 1.0f / den : 0.f;
  for (int channel = lane; channel < HD; channel += 64) {
    float num = 0.f;
    if (channel < vd)
      for (int s0 = 0; s0 < a.splits; s0 += 8) {           // eight runs' values are asked for together
        float x[8], f[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const int s = s0 + j < a.splits ? s0 + j : s0;
          x[j] = runs[(int64_t)s * (HD + 2) + channel];
          f[j] = s0 + j < a.splits ? __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, factor), s)) : 0.f;
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) num += f[j] > 0.f ? x[j] * f[j] : 0.f;
      }
    const float y = num * inv * bt_output_gate(a, tok, head, channel);
    static_cast<bf16_t*>(a.out)[activation_offset<bf16_t>(a.out_rows, a.ldo, tok, head * HD + channel)] = (bf16_t)y;
  }
}

template <int HS, int NV, int NQ>
static int launch(hipStream_t stream, const AttnArgs& a) {
  const int64_t tiles = ((int64_t)a.max_count * a.q_heads + 16 * NQ - 1) / (16 * NQ);
  const int splits = a.splits > 1 ? a.splits : 1;
  if (tiles * a.n_seqs > 0x7fffffff) BT_REFUSE("attention_shared: %lld tiles of rows are too many", (long long)(tiles * a.n_seqs));
  const size_t lds = NQ > 2 ? (size_t)2 * HS * NQ * 64 * sizeof(bf16x8) : 0;
  if (lds > 0) {                                           // with what the kernel holds anyway: beyond what it gets without asking
    static bool raised = false;
    if (!raised) {
      hipError_t err = hipFuncSetAttribute((const void*)attention_shared_kernel<HS, NV, NQ>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      if (err != hipSuccess) BT_REFUSE("attention_shared: cannot get %zu bytes of LDS: %s", lds, hipGetErrorString(err));
      raised = true;
    }
  }
  hipLaunchKernelGGL((attention_shared_kernel<HS, NV, NQ>), dim3((unsigned)(tiles * a.n_seqs), splits), dim3(SHARED_WAVES * 64), lds, stream,
                     a, (int)tiles);
  return bt_check_launch("attention_shared");
}

BT_EXPORT int bt_attention_shared(void* stream, const AttnArgs* args) {
  const AttnArgs& a = *args;
  if (a.n_tokens <= 0 || a.n_seqs <= 0) return BT_OK;
  const int hd = a.kv.head_dim, vd = a.value_dim > 0 ? a.value_dim : hd;
  if (hd <= 0 || hd % 16 != 0 || hd > 768) BT_REFUSE("attention_shared: head size %d must be a multiple of 16 up to 768", hd);
  if (vd > hd || vd % 4 != 0) BT_REFUSE("attention_shared: %d of %d value channels (a multiple of four)", vd, hd);
  if (a.kv.kv_heads != 1 || a.q_heads <= 0) BT_REFUSE("attention_shared: %d query heads on %d cached heads, one is possible", a.q_heads, a.kv.kv_heads);
  if (a.max_count <= 0) BT_REFUSE("attention_shared: max_count %d must be positive", a.max_count);
  if ((int64_t)a.max_count * a.q_heads > 0x3fffffff) BT_REFUSE("attention_shared: too many rows");
  if (a.window < 0 || a.chunk < 0 || a.keep < 0)
    BT_REFUSE("attention_shared: window %d, chunk %d and %d kept positions must not be negative", a.window, a.chunk, a.keep);
  if (!(a.scale > 0.f)) BT_REFUSE("attention_shared: scale %g must be positive", (double)a.scale);
  if (a.form != 0 || a.out_f32) BT_REFUSE("attention_shared: the softmax alone, with bfloat16 results");
  if (const char* wrong = bt_check_form(a)) BT_REFUSE("attention_shared: %s", wrong);
  if (!a.q || !a.out || !a.seq_off || !a.seq_start || !a.kv.blocks || !a.kv.keys || !a.kv.values) BT_REFUSE("attention_shared: missing operand");
  if (a.ldq % 8 != 0 || a.ldo % 4 != 0 || ((uintptr_t)a.q & 15) || ((uintptr_t)a.out & 7) || ((uintptr_t)a.kv.keys & 15) || ((uintptr_t)a.kv.values & 7))
    BT_REFUSE("attention_shared: queries and keys are read 16 bytes at a time, values and results 8");
  if (a.out_rows != 0 && a.out_rows < a.n_tokens) BT_REFUSE("attention_shared: a chunk-major output of %d rows for %d tokens", a.out_rows, a.n_tokens);
  if (a.splits > 1 && (!a.partial || a.splits > 64)) BT_REFUSE("attention_shared: %d runs of keys (at most 64) need a place for their results", a.splits);
  hipStream_t s = (hipStream_t)stream;
  // 64 rows a work-group where there are enough of them for every compute unit, fewer where there are not
  const int64_t most = (int64_t)a.max_count * a.q_heads, all = (int64_t)a.n_tokens * a.q_heads * (a.splits > 1 ? a.splits : 1);
  const int size = most <= 16 ? 1 : most < 64 || all < 64 * SHARED_MANY ? 2 : 4;
  const int v_blocks = (vd + 127) / 128;
  int rc;
#define SHARED_FORM(HS, NV) (size == 1 ? launch<HS, NV, 1>(s, a) : size == 2 ? launch<HS, NV, 2>(s, a) : launch<HS, NV, 4>(s, a))
  if (hd <= 128) rc = SHARED_FORM(2, 1);
  else if (hd <= 256) rc = SHARED_FORM(4, 2);
  else if (hd <= 384) rc = SHARED_FORM(6, 3);
  else if (hd <= 512) rc = SHARED_FORM(8, 4);
  else if (hd <= 576 && v_blocks <= 4) rc = SHARED_FORM(9, 4);
  // (the widest: two blocks of rows would not fit the registers)
  else if (hd <= 640) rc = size < 4 ? launch<10, 5, 1>(s, a) : launch<10, 5, 4>(s, a);
  else rc = size < 4 ? launch<12, 6, 1>(s, a) : launch<12, 6, 4>(s, a);
#undef SHARED_FORM
  if (rc || a.splits <= 1) return rc;
  const int64_t pairs = (int64_t)a.n_tokens * a.q_heads;
  if (pairs > 0x7fffffff) BT_REFUSE("attention_shared: too many rows to join");
  hipLaunchKernelGGL(attention_shared_join_kernel, dim3((unsigned)((pairs + 3) / 4)), dim3(256), 0, s, a);
  return bt_check_launch("attention_shared");
}

BT_EXPORT int bt_attention_shared_call(void* stream, const AttentionCall* c) { return bt_attention_shared(stream, &c->args); }
