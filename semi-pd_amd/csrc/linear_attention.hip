// Linear attention with decays over a pool of per-request state rows (gfx950, wave64).
//
// Rows of the projection hold q [H D], k [H D], v [H E] and an output gate g [H E].  Per head, a matrix S [D, E] from zero, fp32:
//     S_t = diag(alpha_t) S_(t-1) + k_t v_t^T;      o_t = S_t^T q_t * q_scale
// with one of two decays:
//  * per channel: alpha_t [D] = sigmoid(A2 a_t + b)^(1 / tau), a_t [rank] a further column range of the row, A2 [H D, rank];
//  * per head: a constant.
// q, k and v may go through silu first (rounded to the activation type, as a projection of that type would hold them).  Then an RMS
// norm of every head (one weight [E] for all) or of all heads together (weight [H E]), times silu(g) or sigmoid(g).
//
// The state row of a request: S of all heads [H, D, E].  A sequence's first rows start from zero whatever the row holds; otherwise
// the state is read before a launch's rows and written back behind them, so prompts cut into portions, single decode tokens and
// rows that change hands take one path.
//
//  * Prompt batches in bf16, 64 tokens at a time on the matrix cores.  With b_t the running sum of log alpha inside the chunk,
//        o_t = (q_t e^(b_t)) S_in + sum_(s <= t) A_ts v_s,    A_ts = sum_d q_td k_sd e^(b_td - b_sd)
//        S_out = diag(e^(b_last)) S_in + sum_s (k_s e^(b_last - b_s)) v_s^T
//    Everything in front of S and v is independent of the chunks before it: channel_operands_kernel / head_operands_kernel compute
//    it for all (chunk, head) at once and lay it down in the order in which matrix operands are held -- 1 KB per 16 x 32 operand, a
//    lane's 16 bytes at its own place -- and chunk_walk_kernel, a workgroup per (request, head, up to 64 columns of S), goes through
//    the chunks with S in fp32 accumulators, operands coming straight into registers one chunk ahead; half of its waves make the
//    next S while the other half read results out of the one in front.  Decayed q, k, A and S
//    enter a product as their upper 16 bits plus the bf16 of the rest (about 2^-17 relative); sums are fp32.
//    Per-channel decays have no common factor to take out of a sum over d, so a chunk is four tiles of 16 tokens: between
//    tiles the exponents split at a tile's edge into two parts, neither above 0; inside a tile they split at its middle as long as
//    no channel loses more than 2^100 over the tile, and are taken pair by pair where one does.
//  * linear_scan_kernel: every element type and size, token by token, one wave per (request, head, 64 / NS columns of S).
//  * linear_step_kernel: batches of one token per request, a workgroup per (request, head, 64 columns): S is read and written
//    once, 16-byte accesses, every load of a thread in flight before the first is used.
//  * linear_out_kernel: norm, weight and gate.
#include "common.h"
#include "mfma_frag.h"

namespace semipd {

struct LinArgs {
  const void* p; int64_t ld;                              // projection rows
  int64_t q_off, k_off, v_off, g_off;                     // their columns
  int64_t a_off; int rank; const void* a2; const float* a2_bias; float inv_tau;      // per-channel decay (a2 NULL: per head)
  const float* powers;                                    // [H, 65]: a head's decay to the power 0 .. 64
  int act;                                                // q, k, v through silu
  float* work; int64_t wld;                               // fp32 [T, wld]: o [H E]
  float* alpha;                                           // fp32 [T, H D] (token by token, per channel)
  uint8_t* frags; float* keep;                            // operands of a chunk and e^(b_last) [chunks, H, 32 ND] (matrix-core form)
  float* state; int64_t state_ld;                         // fp32 [slots, >= H D E]
  const int64_t* state_indices; const int64_t* seq_lens;
  const int32_t* q_start; const int32_t* q_len;           // [B] or NULL (one row per request)
  int64_t batch, num_tokens;
  int H, D, E;
  float q_scale;
  const void* norm_w; int together; float eps;            // weight of the activation type, [H E] (together) or [E]
  int gate_silu;
  void* out; int64_t out_ld;                              // [T, H E] of the activation type
};

constexpr int kLinChunk = 64;
constexpr float kLinLog2e = 1.4426950408889634f;

__device__ __forceinline__ float lin_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
template <typename T> __device__ __forceinline__ float lin_act(float x, int act) {
  return act ? Elem<T>::to_f(Elem<T>::from_f(x / (1.0f + expf(-x)))) : x;
}
// log2 of sigmoid(x)^(inv_tau); 1 + e rounds once, an error of an ulp of the decay itself
__device__ __forceinline__ float log2_decay(float x, float inv_tau) {
  const float y = x * kLinLog2e;
  return (fminf(y, 0.f) - __builtin_amdgcn_logf(1.0f + __builtin_amdgcn_exp2f(-fabsf(y)))) * inv_tau;
}

// the rows of request b in this launch: first row, how many, position of the first
__device__ __forceinline__ bool linear_rows(const LinArgs& a, int b, int64_t& t0, int64_t& n, int64_t& first_pos) {
  if (a.q_start == nullptr) {
    t0 = b; n = 1; first_pos = a.seq_lens[b] - 1;
  } else {
    t0 = a.q_start[b]; n = a.q_len[b]; first_pos = a.seq_lens[b] - n;
  }
  return n > 0 && first_pos >= 0;
}

// Chunk `idx` of the launch (request after request, each in chunks of 64 rows) -> request and chunk in it; a whole wave asks.
__device__ __forceinline__ bool find_chunk(const LinArgs& a, int64_t idx, int& b, int64_t& c) {
  const int lane = threadIdx.x & 63;
  int64_t before = 0;
  for (int r0 = 0; r0 < (int)a.batch; r0 += 64) {
    const int n = r0 + lane < (int)a.batch ? (a.q_len[r0 + lane] + kLinChunk - 1) / kLinChunk : 0;
    int s = n;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int t = __shfl_up(s, o, 64);
      if (lane >= o) s += t;
    }
    const int total = __shfl(s, 63, 64);
    if (idx < before + total) {
      const uint64_t past = __ballot(before + s > idx);
      const int first = __ffsll((unsigned long long)past) - 1;
      b = r0 + first;
      c = idx - before - (__shfl(s, first, 64) - __shfl(n, first, 64));
      return true;
    }
    before += total;
  }
  return false;
}
// how many chunks the requests in front of b have
__device__ __forceinline__ int64_t chunks_before(const LinArgs& a, int b) {
  const int lane = threadIdx.x & 63;
  int s = 0;
  for (int r = lane; r < b; r += 64) s += (a.q_len[r] + kLinChunk - 1) / kLinChunk;
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) s += __shfl_xor(s, o, 64);
  return s;
}

// x as its upper 16 bits and the bf16 of what they leave of it
__device__ __forceinline__ void hi_lo(float x0, float x1, uint32_t& hi, uint32_t& lo) {
  const uint32_t w0 = __float_as_uint(x0), w1 = __float_as_uint(x1);
  hi = __builtin_amdgcn_perm(w1, w0, 0x07060302u);
  lo = pack2<bf16_t>(x0 - __uint_as_float(w0 & 0xffff0000u), x1 - __uint_as_float(w1 & 0xffff0000u));
}
__device__ __forceinline__ void hi_lo8(const float (&x)[8], Frag16& hi, Frag16& lo) {
#pragma unroll
  for (int u = 0; u < 4; ++u) hi_lo(x[2 * u], x[2 * u + 1], hi.w[u], lo.w[u]);
}
__device__ __forceinline__ void widen8(const Frag16& f, float (&x)[8]) {
#pragma unroll
  for (int u = 0; u < 4; ++u) {
    x[2 * u] = __uint_as_float(f.w[u] << 16);
    x[2 * u + 1] = __uint_as_float(f.w[u] & 0xffff0000u);
  }
}
__device__ __forceinline__ void silu8(Frag16& f) {
  float x[8];
  widen8(f, x);
#pragma unroll
  for (int u = 0; u < 8; ++u) x[u] *= __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-x[u] * kLinLog2e));
#pragma unroll
  for (int u = 0; u < 4; ++u) f.w[u] = pack2<bf16_t>(x[2 * u], x[2 * u + 1]);
}

// ---------------------------------------------------------------------------------- operands of a chunk
// Per (chunk, head), in KB: decayed queries [4 tiles][ND][hi, lo] | decayed keys, transposed [2 ND tiles of d][2][hi, lo] |
// A [4 tiles of queries][2][hi, lo].  An operand's 32 summed-over elements -- tokens of step s, channels of step kk -- are, for
// lanes of group g: 32 s + 4 g .. + 3, then 32 s + 16 + 4 g .. + 3: how the rows of two neighbouring 16-row results lie in a
// lane, so results become operands without changing lanes.
__host__ __device__ constexpr int lin_q_frag(int nd, int tile, int kk) { return (tile * nd + kk) * 2; }
__host__ __device__ constexpr int lin_k_frag(int nd, int dt, int s) { return 8 * nd + (dt * 2 + s) * 2; }
__host__ __device__ constexpr int lin_a_frag(int nd, int tile, int s) { return 16 * nd + (tile * 2 + s) * 2; }
__host__ __device__ constexpr int lin_frags(int nd) { return 16 * nd + 16; }
__host__ __device__ constexpr int lin_row(int nd) { return nd * 64 + 32; }              // bytes of an LDS row of 32 ND bf16 elements

__device__ __forceinline__ void put_frag(uint8_t* base, int idx, const Frag16& f) {
  *reinterpret_cast<uint4*>(base + (int64_t)idx * 1024 + (threadIdx.x & 63) * 16) = f.u;
}
__device__ __forceinline__ uint4 get_frag(const uint8_t* base, int idx) {
  return *reinterpret_cast<const uint4*>(base + (int64_t)idx * 1024 + (threadIdx.x & 63) * 16);
}

// 8 of the 32 elements of a step from a row of memory, in the order above (n a multiple of 4: elements from n on are zero)
__device__ __forceinline__ Frag16 two_pieces(const bf16_t* row, int first, int n) {
  const int g = (threadIdx.x & 63) >> 4, d0 = first + 4 * g, d1 = d0 + 16;
  uint2 a = {0u, 0u}, b = {0u, 0u};
  if (d0 < n) a = *reinterpret_cast<const uint2*>(row + d0);
  if (d1 < n) b = *reinterpret_cast<const uint2*>(row + d1);
  Frag16 f;
  f.u = uint4{a.x, a.y, b.x, b.y};
  return f;
}

// the transposed operand [16 rows][32 tokens] of an LDS tile of token rows; PERMUTED: the rows' elements lie in the order above
template <int STRIDE, bool PERMUTED> __device__ __forceinline__ Frag16 transposed(const uint8_t* tile, int s, int col16) {
  const int lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
  const uint8_t* row = tile + (32 * s + 4 * g + (r >> 2)) * STRIDE +
                       (PERMUTED ? (r & 3) * 16 + (col16 & 1) * 8 + (col16 >> 1) * 64 : (r & 3) * 8 + col16 * 32);
  Frag16 f;
  f.s[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)row);
  f.s[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(row + 16 * STRIDE));
  return f;
}

// tiles of A (rows: keys, columns: this wave's queries) as operands over the keys; tiles behind the queries' own are zero
__device__ __forceinline__ void put_weights(uint8_t* base, int nd, int tile, const f32x4 (&w)[4]) {
#pragma unroll
  for (int s = 0; s < 2; ++s) {
    if (2 * s > tile) break;
    Frag16 hi, lo;
#pragma unroll
    for (int half = 0; half < 2; ++half) {
      hi_lo(w[2 * s + half][0], w[2 * s + half][1], hi.w[2 * half], lo.w[2 * half]);
      hi_lo(w[2 * s + half][2], w[2 * s + half][3], hi.w[2 * half + 1], lo.w[2 * half + 1]);
    }
    put_frag(base, lin_a_frag(nd, tile, s), hi);
    put_frag(base, lin_a_frag(nd, tile, s) + 1, lo);
  }
}

// keys of the chunk in LDS (upper and lower parts) -> transposed operands, ND / 2 tiles of d per wave
template <int ND> __device__ __forceinline__ void put_keys(uint8_t* base, const uint8_t* kh, const uint8_t* kl) {
  const int wave = threadIdx.x >> 6;
#pragma unroll
  for (int i = 0; i < ND / 2; ++i) {
    const int dt = (ND / 2) * wave + i;
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      put_frag(base, lin_k_frag(ND, dt, s), transposed<lin_row(ND), true>(kh, s, dt));
      put_frag(base, lin_k_frag(ND, dt, s) + 1, transposed<lin_row(ND), true>(kl, s, dt));
    }
  }
}

template <int CTRL> __device__ __forceinline__ float dpp(float x) {       // row operations inside 16 lanes, 0 where nothing comes in
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), CTRL, 0xf, 0xf, false));
}
__device__ __forceinline__ float sum_up_to(float x) {                     // inclusive running sum over 16 lanes
  x += dpp<0x111>(x);
  x += dpp<0x112>(x);
  x += dpp<0x114>(x);
  return x + dpp<0x118>(x);
}
template <int LANE> __device__ __forceinline__ float of_lane(float x) { return dpp<0x150 + LANE>(x); }      // lane LANE of the 16 (row_newbcast)

template <int ND> constexpr size_t channel_lds() { return 2 * (size_t)kLinChunk * lin_row(ND) + 4 * 32 * ND * sizeof(float); }

template <int ND>          // key sizes up to 32 ND; wave = tile of 16 tokens, lane r of 16 = token
__global__ void __launch_bounds__(256, 2) channel_operands_kernel(LinArgs a) {
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
  constexpr int DP = 32 * ND, RS = lin_row(ND);
  uint8_t* kh = lds;                                                    // keys, upper and lower parts [64][RS]
  uint8_t* kl = lds + kLinChunk * RS;
  float* loss = reinterpret_cast<float*>(lds + 2 * kLinChunk * RS);     // what a channel keeps over a whole tile [4][DP], in the operands' order
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, g = lane >> 4;
  const int h = blockIdx.y, D = a.D, rank = a.rank;
  int b;
  int64_t c;
  if (!find_chunk(a, blockIdx.x, b, c)) return;
  const int64_t c0 = c * kLinChunk;
  const int cnt = (int)(a.q_len[b] - c0 < kLinChunk ? a.q_len[b] - c0 : kLinChunk);
  const int row = 16 * wave + r;
  const bf16_t* pr = (const bf16_t*)a.p + (a.q_start[b] + c0 + (row < cnt ? row : cnt - 1)) * a.ld;
  uint8_t* out = a.frags + ((int64_t)blockIdx.x * a.H + h) * lin_frags(ND) * 1024;
  const bf16_t* a2 = (const bf16_t*)a.a2 + (int64_t)h * D * rank;
  const bool wide = rank % 4 == 0 && (a.a_off & 3) == 0 && ((uintptr_t)a.a2 & 7) == 0;
  auto rank_piece = [&](const bf16_t* src, int first) {                 // 32 elements of a row of A1 h or A2
    if (wide) return two_pieces(src, first, rank);
    Frag16 f;
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      const int i = first + 4 * g + (u & 3) + (u >> 2) * 16;
      f.e[u] = i < rank ? src[i].v : (uint16_t)0;
    }
    return f;
  };
  const Frag16 a1 = rank_piece(pr + a.a_off, 0);

  float q8[ND][8], k8[ND][8];              // queries from their tile's start, keys to their tile's end
  f32x4 own = {0.f, 0.f, 0.f, 0.f};        // A inside the tile: key 4 g + i, query r
#pragma unroll
  for (int kk = 0; kk < ND; ++kk) {
    // running sums of the log2 decays: rows = channels 32 kk + 16 half + 4 g + i, column = this lane's token
    float cs[8], q[8], k[8];
#pragma unroll
    for (int half = 0; half < 2; ++half) {
      const int dr = 32 * kk + 16 * half + r, dz = 32 * kk + 16 * half + 4 * g;
      const bf16_t* w = a2 + (int64_t)(dr < D ? dr : 0) * rank;
      float bias[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) bias[i] = dz < D ? a.a2_bias[h * D + dz + i] : 0.f;
      f32x4 z = {0.f, 0.f, 0.f, 0.f};
      z = mma16<bf16_t>(rank_piece(w, 0), a1, z);
      for (int r0 = 32; r0 < rank; r0 += 32) z = mma16<bf16_t>(rank_piece(w, r0), rank_piece(pr + a.a_off, r0), z);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const bool there = row < cnt && dz < D;
        const float x = there ? log2_decay(z[i] + bias[i], a.inv_tau) : 0.f;
        cs[4 * half + i] = sum_up_to(x);
      }
    }
    Frag16 qf = two_pieces(pr + a.q_off + (int64_t)h * D, 32 * kk, D), kf = two_pieces(pr + a.k_off + (int64_t)h * D, 32 * kk, row < cnt ? D : 0);
    if (a.act) {
      silu8(qf);
      silu8(kf);
    }
    widen8(qf, q);
    widen8(kf, k);
    float total[8];
    bool gentle = true;                    // none of these channels loses more than 2^100 over the tile
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      total[u] = of_lane<15>(cs[u]);
      gentle = gentle && total[u] > -100.f;
    }
    if (r == 0) {
      float* t = loss + wave * DP + 32 * kk + 8 * g;
#pragma unroll
      for (int u = 0; u < 8; ++u) t[u] = __builtin_amdgcn_exp2f(total[u]);
    }
    if (__all(gentle)) {                   // the tile's own pairs: both sides relative to the tile's eighth token
      Frag16 qh, ql, ah, al;
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const float mid = of_lane<7>(cs[u]), e = __builtin_amdgcn_exp2f(cs[u] - mid);
        q[u] *= e;
        k[u] *= __builtin_amdgcn_rcpf(e);
        q8[kk][u] = q[u] * __builtin_amdgcn_exp2f(mid);
        k8[kk][u] = k[u] * __builtin_amdgcn_exp2f(total[u] - mid);
      }
      hi_lo8(q, qh, ql);
      hi_lo8(k, ah, al);
      own = mma16<bf16_t>(ah, qh, own);
      own = mma16<bf16_t>(al, qh, own);
      own = mma16<bf16_t>(ah, ql, own);
    } else {                               // pair by pair
#pragma unroll 1
      for (int j = 0; j < 16; ++j) {
        float part = 0.f;
#pragma unroll
        for (int u = 0; u < 8; ++u) {
          const float cj = __shfl(cs[u], (lane & 48) | j, 64), kj = __shfl(k[u], (lane & 48) | j, 64);
          part += q[u] * kj * __builtin_amdgcn_exp2f(fminf(cs[u] - cj, 0.f));
        }
        part += __shfl_xor(part, 16, 64);
        part += __shfl_xor(part, 32, 64);
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (4 * g + i == j) own[i] += part;
      }
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        q8[kk][u] = q[u] * __builtin_amdgcn_exp2f(cs[u]);
        k8[kk][u] = k[u] * __builtin_amdgcn_exp2f(total[u] - cs[u]);
      }
    }
    Frag16 hi, lo;
    hi_lo8(k8[kk], hi, lo);
    *reinterpret_cast<uint4*>(kh + row * RS + (32 * kk + 8 * g) * 2) = hi.u;
    *reinterpret_cast<uint4*>(kl + row * RS + (32 * kk + 8 * g) * 2) = lo.u;
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) own[i] = 4 * g + i <= r ? own[i] : 0.f;
  __syncthreads();
  if (tid < DP) {
    const int p32 = tid & 31, d = (tid & ~31) + ((p32 >> 2) & 1) * 16 + (p32 >> 3) * 4 + (p32 & 3);
    a.keep[((int64_t)blockIdx.x * a.H + h) * DP + d] = (loss[tid] * loss[DP + tid]) * (loss[2 * DP + tid] * loss[3 * DP + tid]);
  }
  auto read8 = [&](int tile, int kk, float (&x)[8]) {
    const float* src = loss + tile * DP + 32 * kk + 8 * g;
    const float4 lo = *reinterpret_cast<const float4*>(src), hi = *reinterpret_cast<const float4*>(src + 4);
    x[0] = lo.x; x[1] = lo.y; x[2] = lo.z; x[3] = lo.w; x[4] = hi.x; x[5] = hi.y; x[6] = hi.z; x[7] = hi.w;
  };
  // tiles in front, from the nearest on: keys relative to their tile's end, queries brought to the end of that tile, and past the
  // first tile to the chunk's start
  f32x4 back[3];                           // tile wave - 1 - x
#pragma unroll
  for (int x = 0; x < 3; ++x) back[x] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int kk = 0; kk < ND; ++kk) {
    Frag16 hi, lo;
    float t[8];
#pragma unroll
    for (int x = 0; x < 3; ++x) {
      const int J = wave - 1 - x;
      if (J < 0) break;
      Frag16 ah, al;
      ah.u = *reinterpret_cast<const uint4*>(kh + (16 * J + r) * RS + (32 * kk + 8 * g) * 2);
      al.u = *reinterpret_cast<const uint4*>(kl + (16 * J + r) * RS + (32 * kk + 8 * g) * 2);
      hi_lo8(q8[kk], hi, lo);
      back[x] = mma16<bf16_t>(ah, hi, back[x]);
      back[x] = mma16<bf16_t>(al, hi, back[x]);
      back[x] = mma16<bf16_t>(ah, lo, back[x]);
      read8(J, kk, t);
#pragma unroll
      for (int u = 0; u < 8; ++u) q8[kk][u] *= t[u];
    }
    hi_lo8(q8[kk], hi, lo);
    put_frag(out, lin_q_frag(ND, wave, kk), hi);
    put_frag(out, lin_q_frag(ND, wave, kk) + 1, lo);
    for (int s = wave + 1; s < 4; ++s) {   // keys to the chunk's end
      read8(s, kk, t);
#pragma unroll
      for (int u = 0; u < 8; ++u) k8[kk][u] *= t[u];
    }
  }
  f32x4 w[4];
#pragma unroll
  for (int kt = 0; kt < 4; ++kt) {
    w[kt] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (kt == wave) w[kt] = own;
#pragma unroll
    for (int x = 0; x < 3; ++x)
      if (kt == wave - 1 - x) w[kt] = back[x];
  }
  put_weights(out, ND, wave, w);
  __syncthreads();
#pragma unroll
  for (int kk = 0; kk < ND; ++kk) {
    Frag16 hi, lo;
    hi_lo8(k8[kk], hi, lo);
    *reinterpret_cast<uint4*>(kh + row * RS + (32 * kk + 8 * g) * 2) = hi.u;
    *reinterpret_cast<uint4*>(kl + row * RS + (32 * kk + 8 * g) * 2) = lo.u;
  }
  __syncthreads();
  put_keys<ND>(out, kh, kl);
}

template <int ND>          // one decay per head: it factors out of the sum over d
__global__ void __launch_bounds__(256, 2) head_operands_kernel(LinArgs a) {
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
  constexpr int DP = 32 * ND, RS = lin_row(ND);
  __shared__ float pw[kLinChunk + 1];
  uint8_t* kh = lds;
  uint8_t* kl = lds + kLinChunk * RS;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, g = lane >> 4;
  const int h = blockIdx.y, D = a.D;
  int b;
  int64_t c;
  if (!find_chunk(a, blockIdx.x, b, c)) return;
  const int64_t c0 = c * kLinChunk;
  const int cnt = (int)(a.q_len[b] - c0 < kLinChunk ? a.q_len[b] - c0 : kLinChunk);
  uint8_t* out = a.frags + ((int64_t)blockIdx.x * a.H + h) * lin_frags(ND) * 1024;
  if (tid <= kLinChunk) pw[tid] = a.powers[h * (kLinChunk + 1) + tid];
  const int row = 16 * wave + r;
  const bf16_t* pr = (const bf16_t*)a.p + (a.q_start[b] + c0 + (row < cnt ? row : cnt - 1)) * a.ld + (int64_t)h * D;
  Frag16 qf[ND], kf[ND];
#pragma unroll
  for (int kk = 0; kk < ND; ++kk) {
    qf[kk] = two_pieces(pr + a.q_off, 32 * kk, D);
    kf[kk] = two_pieces(pr + a.k_off, 32 * kk, row < cnt ? D : 0);
  }
  if (a.act) {
#pragma unroll
    for (int kk = 0; kk < ND; ++kk) {
      silu8(qf[kk]);
      silu8(kf[kk]);
    }
  }
#pragma unroll
  for (int kk = 0; kk < ND; ++kk) *reinterpret_cast<uint4*>(kh + row * RS + (32 * kk + 8 * g) * 2) = kf[kk].u;
  __syncthreads();
  if (tid < DP) a.keep[((int64_t)blockIdx.x * a.H + h) * DP + tid] = pw[cnt];
  const float qw = pw[row + 1], kw = row < cnt ? pw[cnt - 1 - row] : 0.f;
  f32x4 w[4];
#pragma unroll
  for (int kt = 0; kt < 4; ++kt) w[kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int kk = 0; kk < ND; ++kk) {
    float x[8];
    Frag16 hi, lo;
    widen8(qf[kk], x);
#pragma unroll
    for (int u = 0; u < 8; ++u) x[u] *= qw;
    hi_lo8(x, hi, lo);
    put_frag(out, lin_q_frag(ND, wave, kk), hi);
    put_frag(out, lin_q_frag(ND, wave, kk) + 1, lo);
#pragma unroll
    for (int kt = 0; kt < 4; ++kt) {
      if (kt > wave) break;
      Frag16 f;
      f.u = *reinterpret_cast<const uint4*>(kh + (16 * kt + r) * RS + (32 * kk + 8 * g) * 2);
      w[kt] = mma16<bf16_t>(f, qf[kk], w[kt]);
    }
  }
#pragma unroll
  for (int kt = 0; kt < 4; ++kt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int back = row - (16 * kt + 4 * g + i);
      w[kt][i] = back >= 0 ? w[kt][i] * pw[back < 0 ? 0 : back] : 0.f;
    }
  put_weights(out, ND, wave, w);
  __syncthreads();
#pragma unroll
  for (int kk = 0; kk < ND; ++kk) {
    float x[8];
    Frag16 hi, lo;
    widen8(kf[kk], x);
#pragma unroll
    for (int u = 0; u < 8; ++u) x[u] *= kw;
    hi_lo8(x, hi, lo);
    *reinterpret_cast<uint4*>(kh + row * RS + (32 * kk + 8 * g) * 2) = hi.u;
    *reinterpret_cast<uint4*>(kl + row * RS + (32 * kk + 8 * g) * 2) = lo.u;
  }
  __syncthreads();
  put_keys<ND>(out, kh, kl);
}

// ---------------------------------------------------------------------------------- the walk over a request's chunks
// Eight waves with two jobs.  Waves 4 .. 7 carry S in fp32 accumulators from chunk to chunk: S <- diag(e^(b_last)) S + K^T V, then S
// as upper and lower bf16 parts into LDS; they also bring the chunk's values there.  Waves 0 .. 3, one per 16 queries, turn the S
// that the chunk found and its values into results.  S and the values have two places each, so while results of a chunk are
// computed the next S is already being made, with one barrier per chunk; both jobs' operands come from memory straight into
// registers, one chunk ahead.
template <int EC> constexpr int lin_v_row() { return EC * 32 + 32; }
template <int ND, int EC> constexpr size_t walk_lds() { return 4 * (size_t)(16 * EC) * lin_row(ND) + 2 * (size_t)kLinChunk * lin_v_row<EC>(); }

template <int ND, int EC>          // key sizes up to 32 ND; 16 EC columns of S per workgroup
__global__ void __launch_bounds__(512, 2) chunk_walk_kernel(LinArgs a) {
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
  constexpr int RS = lin_row(ND), VS = lin_v_row<EC>(), DP = 32 * ND, COLS = 16 * EC;
  constexpr int S_PART = COLS * RS, S_BUF = 2 * S_PART, V_BUF = kLinChunk * VS;
  uint8_t* s_lds = lds;                                                  // [2][upper, lower][COLS][RS]
  uint8_t* v_lds = lds + 2 * S_BUF;                                      // [2][64][VS]
  const int tid = threadIdx.x, lane = tid & 63, r = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int H = a.H, D = a.D, E = a.E;
  const int slices = (E + COLS - 1) / COLS;
  // consecutive workgroup ids go round the eight XCDs: an XCD takes a contiguous range of items, so the slices of a head --
  // which read the same operands -- share an L2 (gridDim.x is a multiple of 8)
  const int64_t n_items = gridDim.x, item = (int64_t)(blockIdx.x & 7) * (n_items >> 3) + (blockIdx.x >> 3);
  if (item >= a.batch * H * slices) return;
  const int sl = (int)(item % slices), h = (int)(item / slices % H), b = (int)(item / slices / H);
  int64_t t0, n, first_pos;
  if (!linear_rows(a, b, t0, n, first_pos)) return;
  const int e0 = sl * COLS;
  const int64_t chunk0 = chunks_before(a, b);
  const int chunks = (int)((n + kLinChunk - 1) / kLinChunk);             // every wave passes 1 barrier per chunk
  const int64_t frag_step = (int64_t)H * lin_frags(ND) * 1024;
  const uint8_t* fr = a.frags + (chunk0 * H + h) * (int64_t)lin_frags(ND) * 1024;

  if (wave < 4) {
    // ---- results of queries 16 wave + r, all columns
    const int qt = wave;
    float* work = a.work + (t0 + 16 * qt + r) * a.wld + (int64_t)h * E + e0;
    Frag16 qf[ND][2], wf[2][2];
    auto fetch_q = [&](const uint8_t* f) {
#pragma unroll
      for (int kk = 0; kk < ND; ++kk) {
        qf[kk][0].u = get_frag(f, lin_q_frag(ND, qt, kk));
        qf[kk][1].u = get_frag(f, lin_q_frag(ND, qt, kk) + 1);
      }
    };
    auto fetch_w = [&](const uint8_t* f) {
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        if (2 * s > qt) break;
        wf[s][0].u = get_frag(f, lin_a_frag(ND, qt, s));
        wf[s][1].u = get_frag(f, lin_a_frag(ND, qt, s) + 1);
      }
    };
    fetch_q(fr);
    fetch_w(fr);
    for (int c = 0; c < chunks; ++c) {
      const int64_t left = n - (int64_t)c * kLinChunk - 16 * qt;         // rows of this tile that are there
      const bool more = c + 1 < chunks;
      const uint8_t* s_hi = s_lds + (c & 1) * S_BUF;
      const uint8_t* s_lo = s_hi + S_PART;
      const uint8_t* v_in = v_lds + (c & 1) * V_BUF;
      fr += frag_step;
      __syncthreads();
      f32x4 o[EC];
#pragma unroll
      for (int et = 0; et < EC; ++et) o[et] = f32x4{0.f, 0.f, 0.f, 0.f};
      // the operands of the next 32 elements are on their way out of LDS during a product
      Frag16 sa[2][EC][2];
      auto load = [&](int kk, Frag16 (&x)[EC][2]) {
#pragma unroll
        for (int et = 0; et < EC; ++et) {
          const int off = (16 * et + r) * RS + g * 16 + kk * 64;
          x[et][0].u = *reinterpret_cast<const uint4*>(s_hi + off);
          x[et][1].u = *reinterpret_cast<const uint4*>(s_lo + off);
        }
      };
      load(0, sa[0]);
#pragma unroll
      for (int kk = 0; kk < ND; ++kk) {
        if (kk + 1 < ND) load(kk + 1, sa[(kk + 1) & 1]);
        __builtin_amdgcn_sched_barrier(0);
        Frag16(&x)[EC][2] = sa[kk & 1];
#pragma unroll
        for (int et = 0; et < EC; ++et) o[et] = mma16<bf16_t>(x[et][0], qf[kk][0], o[et]);
#pragma unroll
        for (int et = 0; et < EC; ++et) o[et] = mma16<bf16_t>(x[et][1], qf[kk][0], o[et]);
#pragma unroll
        for (int et = 0; et < EC; ++et) o[et] = mma16<bf16_t>(x[et][0], qf[kk][1], o[et]);
        __builtin_amdgcn_sched_barrier(0);
      }
      if (more) fetch_q(fr);
      // the chunk's own tokens
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        if (2 * s > qt) break;
        Frag16 v[EC];
#pragma unroll
        for (int et = 0; et < EC; ++et) v[et] = transposed<VS, false>(v_in, s, et);
#pragma unroll
        for (int et = 0; et < EC; ++et) o[et] = mma16<bf16_t>(v[et], wf[s][0], o[et]);
#pragma unroll
        for (int et = 0; et < EC; ++et) o[et] = mma16<bf16_t>(v[et], wf[s][1], o[et]);
      }
      if (more) fetch_w(fr);
      if (r < left) {
#pragma unroll
        for (int et = 0; et < EC; ++et) {
          const int e = 16 * et + 4 * g;
          if (e0 + e < E) *reinterpret_cast<float4*>(work + e) =
              float4{o[et][0] * a.q_scale, o[et][1] * a.q_scale, o[et][2] * a.q_scale, o[et][3] * a.q_scale};
        }
      }
      work += kLinChunk * a.wld;
    }
    return;
  }

  // ---- S: rows d = 16 (dt0 + dt) + 4 g + i, column e0 + 16 et + r
  constexpr int DTW = ND / 2, VP = EC / 2;
  const int dt0 = (wave - 4) * DTW, vt = tid - 256;
  const bool fresh = first_pos == 0;
  float* S = a.state + a.state_indices[b] * a.state_ld + (int64_t)h * D * E + e0;
  const int64_t keep_step = (int64_t)H * DP;
  const float* keep = a.keep + (chunk0 * H + h) * DP;
  const bf16_t* vp = (const bf16_t*)a.p + t0 * a.ld + a.v_off + (int64_t)h * E;
  f32x4 acc[DTW][EC];
#pragma unroll
  for (int dt = 0; dt < DTW; ++dt)
#pragma unroll
    for (int et = 0; et < EC; ++et)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = 16 * (dt0 + dt) + 4 * g + i, e = 16 * et + r;
        acc[dt][et][i] = (!fresh && d < D && e0 + e < E) ? S[(int64_t)d * E + e] : 0.f;
      }
  Frag16 kf[DTW][2][2], vr[VP];
  float4 kp[DTW];
  // values, in 16-byte pieces (past the end the last row, past E the first columns: finite numbers that meet zero weights or
  // columns that are not kept)
  auto fetch_v = [&](int c) {
    const int64_t base = (int64_t)c * kLinChunk, last = n - 1 - base;
#pragma unroll
    for (int i = 0; i < VP; ++i) {
      const int x = vt + 256 * i, row = x / (2 * EC), e = e0 + (x % (2 * EC)) * 8;
      vr[i].u = *reinterpret_cast<const uint4*>(vp + (base + (row < last ? row : last)) * a.ld + (e < E ? e : 0));
    }
  };
  auto lay_v = [&](uint8_t* v_out) {
#pragma unroll
    for (int i = 0; i < VP; ++i) {
      const int x = vt + 256 * i;
      if (a.act) silu8(vr[i]);
      *reinterpret_cast<uint4*>(v_out + x / (2 * EC) * VS + (x % (2 * EC)) * 16) = vr[i].u;
    }
  };
  auto lay_s = [&](uint8_t* s_out) {
#pragma unroll
    for (int dt = 0; dt < DTW; ++dt) {
      const int at = ((dt0 + dt) >> 1) * 64 + 16 * g + ((dt0 + dt) & 1) * 8;      // in the operands' order
#pragma unroll
      for (int et = 0; et < EC; ++et) {
        uint2 hi, lo;
        hi_lo(acc[dt][et][0], acc[dt][et][1], hi.x, lo.x);
        hi_lo(acc[dt][et][2], acc[dt][et][3], hi.y, lo.y);
        *reinterpret_cast<uint2*>(s_out + (16 * et + r) * RS + at) = hi;
        *reinterpret_cast<uint2*>(s_out + S_PART + (16 * et + r) * RS + at) = lo;
      }
    }
  };
  auto fetch_k = [&](const uint8_t* f, const float* kd) {
#pragma unroll
    for (int dt = 0; dt < DTW; ++dt) {
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        kf[dt][s][0].u = get_frag(f, lin_k_frag(ND, dt0 + dt, s));
        kf[dt][s][1].u = get_frag(f, lin_k_frag(ND, dt0 + dt, s) + 1);
      }
      kp[dt] = *reinterpret_cast<const float4*>(kd + 16 * (dt0 + dt) + 4 * g);
    }
  };
  fetch_v(0);
  fetch_k(fr, keep);
  lay_s(s_lds);
  lay_v(v_lds);
  if (chunks > 1) fetch_v(1);
  for (int c = 0; c < chunks; ++c) {
    const bool more = c + 1 < chunks;
    const uint8_t* v_in = v_lds + (c & 1) * V_BUF;
    fr += frag_step;
    keep += keep_step;
    __syncthreads();                     // results of the chunk in front are done with the other two places
    if (more) {
      lay_v(v_lds + ((c + 1) & 1) * V_BUF);
      if (c + 2 < chunks) fetch_v(c + 2);
    }
#pragma unroll
    for (int dt = 0; dt < DTW; ++dt)
#pragma unroll
      for (int et = 0; et < EC; ++et) {
        acc[dt][et][0] *= kp[dt].x;
        acc[dt][et][1] *= kp[dt].y;
        acc[dt][et][2] *= kp[dt].z;
        acc[dt][et][3] *= kp[dt].w;
      }
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      Frag16 v[EC];
#pragma unroll
      for (int et = 0; et < EC; ++et) v[et] = transposed<VS, false>(v_in, s, et);
#pragma unroll
      for (int dt = 0; dt < DTW; ++dt)
#pragma unroll
        for (int et = 0; et < EC; ++et) acc[dt][et] = mma16<bf16_t>(kf[dt][s][0], v[et], acc[dt][et]);
#pragma unroll
      for (int dt = 0; dt < DTW; ++dt)
#pragma unroll
        for (int et = 0; et < EC; ++et) acc[dt][et] = mma16<bf16_t>(kf[dt][s][1], v[et], acc[dt][et]);
    }
    if (more) {
      fetch_k(fr, keep);
      lay_s(s_lds + ((c + 1) & 1) * S_BUF);
    }
  }
#pragma unroll
  for (int dt = 0; dt < DTW; ++dt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * (dt0 + dt) + 4 * g + i;
      if (d >= D) continue;
#pragma unroll
      for (int et = 0; et < EC; ++et) {
        const int e = 16 * et + r;
        if (e0 + e < E) S[(int64_t)d * E + e] = acc[dt][et][i];
      }
    }
}

// ---------------------------------------------------------------------------------- token by token, any type and size
// decay of (token, head, channel), a thread each
template <typename T>
__device__ __forceinline__ float channel_decay(const LinArgs& a, const T* row, int64_t hd) {
  float z = a.a2_bias[hd];
  const T* w = (const T*)a.a2 + hd * a.rank;
  const T* x = row + a.a_off;
  constexpr int V = Elem<T>::kVec;
  if (a.rank % V == 0 && ((((uintptr_t)a.a2) | ((uintptr_t)x)) & 15) == 0) {
    for (int i = 0; i < a.rank; i += V) {
      const Vec16<T> wv = load16(w + i), xv = load16(x + i);
#pragma unroll
      for (int u = 0; u < V; ++u) z += Elem<T>::to_f(xv.e[u]) * Elem<T>::to_f(wv.e[u]);
    }
  } else {
    for (int i = 0; i < a.rank; ++i) z += Elem<T>::to_f(x[i]) * Elem<T>::to_f(w[i]);
  }
  return expf((fminf(z, 0.f) - log1pf(expf(-fabsf(z)))) * a.inv_tau);
}
template <typename T>
__global__ void __launch_bounds__(256) channel_decay_kernel(LinArgs a) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x, hd = (int64_t)a.H * a.D;
  if (i >= a.num_tokens * hd) return;
  a.alpha[i] = channel_decay<T>(a, (const T*)a.p + i / hd * a.ld, i % hd);
}

// A column of S lives in the registers of NS adjacent lanes, NPT rows each.
template <typename T, int NPT, int NS>
__global__ void __launch_bounds__(64) linear_scan_kernel(LinArgs a, int stage) {
  extern __shared__ __attribute__((aligned(16))) float scan_l[];      // per staged token: q [NP] | k [NP] | decay [NP] | v of the block's columns
  constexpr int NP = NPT * NS, COLS = 64 / NS, TOK = 3 * NP + COLS;
  const int lane = threadIdx.x, H = a.H, D = a.D, E = a.E;
  const int eblocks = (E + COLS - 1) / COLS;
  int64_t id = blockIdx.x;
  const int eb = (int)(id % eblocks); id /= eblocks;
  const int h = (int)(id % H), b = (int)(id / H);
  int64_t t0, n, first_pos;
  if (!linear_rows(a, b, t0, n, first_pos)) return;
  const bool fresh = first_pos == 0;
  const int col = lane / NS, ns = lane % NS, e = eb * COLS + col, d0 = ns * NPT;
  const bool e_ok = e < E;
  float* base = a.state + a.state_indices[b] * a.state_ld + (int64_t)h * D * E + e;
  float S[NPT];
#pragma unroll
  for (int i = 0; i < NPT; ++i) S[i] = (!fresh && e_ok && d0 + i < D) ? base[(int64_t)(d0 + i) * E] : 0.f;
  const float fixed = a.a2 ? 0.f : a.powers[h * (kLinChunk + 1) + 1];
  const T* p = (const T*)a.p;
  for (int64_t s0 = 0; s0 < n; s0 += stage) {
    const int cnt = (int)(n - s0 < stage ? n - s0 : stage);
    __syncthreads();
    for (int it = lane; it < cnt * TOK; it += 64) {
      const int k = it / TOK, x = it % TOK;
      const int64_t t = t0 + s0 + k;
      const T* row = p + t * a.ld;
      float v = 0.f;
      if (x < NP) {
        if (x < D) v = lin_act<T>(Elem<T>::to_f(row[a.q_off + (int64_t)h * D + x]), a.act);
      } else if (x < 2 * NP) {
        if (x - NP < D) v = lin_act<T>(Elem<T>::to_f(row[a.k_off + (int64_t)h * D + x - NP]), a.act);
      } else if (x < 3 * NP) {
        if (x - 2 * NP < D) v = a.a2 ? a.alpha[(t * H + h) * D + x - 2 * NP] : fixed;
      } else {
        const int ee = eb * COLS + x - 3 * NP;
        if (ee < E) v = lin_act<T>(Elem<T>::to_f(row[a.v_off + (int64_t)h * E + ee]), a.act);
      }
      scan_l[it] = v;
    }
    __syncthreads();
    for (int k = 0; k < cnt; ++k) {
      const float* l = scan_l + k * TOK;
      const float v = l[3 * NP + col];
      float y = 0.f;
#pragma unroll
      for (int i = 0; i < NPT; ++i) {
        S[i] = l[2 * NP + d0 + i] * S[i] + l[NP + d0 + i] * v;
        y += S[i] * l[d0 + i];
      }
#pragma unroll
      for (int o = 1; o < NS; o <<= 1) y += __shfl_xor(y, o, 64);
      if (ns == 0 && e_ok) a.work[(t0 + s0 + k) * a.wld + (int64_t)h * E + e] = y * a.q_scale;
    }
  }
  if (e_ok) {
#pragma unroll
    for (int i = 0; i < NPT; ++i)
      if (d0 + i < D) base[(int64_t)(d0 + i) * E] = S[i];
  }
}

// ---------------------------------------------------------------------------------- one token per request
// Thread (column group, row group): VEC adjacent columns, every 16th row of S.
template <typename T, int VEC>
__global__ void __launch_bounds__(256) linear_step_kernel(LinArgs a) {
  extern __shared__ __attribute__((aligned(16))) float step_l[];     // q [D] | k [D] | decay [D] | partial sums [16][16 VEC]
  constexpr int COLS = 16 * VEC, BATCH = 16;
  const int tid = threadIdx.x, H = a.H, D = a.D, E = a.E;
  const int b = blockIdx.z, h = blockIdx.y, e0 = blockIdx.x * COLS;
  const int64_t first_pos = a.seq_lens[b] - 1;
  if (first_pos < 0) return;
  const bool fresh = first_pos == 0;
  const T* row = (const T*)a.p + (int64_t)b * a.ld;
  float* stS = a.state + a.state_indices[b] * a.state_ld + (int64_t)h * D * E;
  float* ql = step_l;
  float* kl = step_l + D;
  float* al = step_l + 2 * D;
  float* part = step_l + (3 * D + 3) / 4 * 4;
  const int cg = tid & 15, rg = tid >> 4, e = e0 + cg * VEC;
  const bool e_ok = e < E;
  // the first BATCH rows' state is asked for before anything waits
  float S[BATCH][VEC];
  auto load = [&](int i0) {
#pragma unroll
    for (int i = 0; i < BATCH; ++i) {
      const int d = rg + 16 * (i0 + i);
      if (!fresh && e_ok && d < D) {
        if constexpr (VEC == 4) {
          const float4 x = *reinterpret_cast<const float4*>(stS + (int64_t)d * E + e);
          S[i][0] = x.x; S[i][1] = x.y; S[i][2] = x.z; S[i][3] = x.w;
        } else {
          S[i][0] = stS[(int64_t)d * E + e];
        }
      } else {
#pragma unroll
        for (int u = 0; u < VEC; ++u) S[i][u] = 0.f;
      }
    }
  };
  load(0);
  const float fixed = a.a2 ? 0.f : a.powers[h * (kLinChunk + 1) + 1];
  for (int d = tid; d < D; d += 256) {
    ql[d] = lin_act<T>(Elem<T>::to_f(row[a.q_off + (int64_t)h * D + d]), a.act);
    kl[d] = lin_act<T>(Elem<T>::to_f(row[a.k_off + (int64_t)h * D + d]), a.act);
    al[d] = a.a2 ? channel_decay<T>(a, row, (int64_t)h * D + d) : fixed;
  }
  float v[VEC], y[VEC];
#pragma unroll
  for (int u = 0; u < VEC; ++u) {
    v[u] = e_ok ? lin_act<T>(Elem<T>::to_f(row[a.v_off + (int64_t)h * E + e + u]), a.act) : 0.f;
    y[u] = 0.f;
  }
  __syncthreads();
  for (int i0 = 0; 16 * i0 < D; i0 += BATCH) {
    if (i0 > 0) load(i0);
#pragma unroll
    for (int i = 0; i < BATCH; ++i) {
      const int d = rg + 16 * (i0 + i);
      if (d < D) {
        const float kd = kl[d], qd = ql[d], keep = al[d];
#pragma unroll
        for (int u = 0; u < VEC; ++u) {
          S[i][u] = keep * S[i][u] + kd * v[u];
          y[u] += S[i][u] * qd;
        }
        if (e_ok) {
          if constexpr (VEC == 4)
            *reinterpret_cast<float4*>(stS + (int64_t)d * E + e) = float4{S[i][0], S[i][1], S[i][2], S[i][3]};
          else
            stS[(int64_t)d * E + e] = S[i][0];
        }
      }
    }
  }
#pragma unroll
  for (int u = 0; u < VEC; ++u) part[rg * COLS + cg * VEC + u] = y[u];
  __syncthreads();
  if (tid < COLS && e0 + tid < E) {
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) s += part[i * COLS + tid];
    a.work[(int64_t)b * a.wld + (int64_t)h * E + e0 + tid] = s * a.q_scale;
  }
}

// ---------------------------------------------------------------------------------- norm, weight, gate
// WAVES waves (1: four groups a workgroup, 4: one) normalise a group: a head, or all heads of a row.
template <typename T, int VEC, int WAVES>
__global__ void __launch_bounds__(256) linear_out_kernel(LinArgs a) {
  __shared__ float red[16];
  constexpr int NR = 4, STEP = 64 * WAVES * VEC;      // pieces of VEC elements a lane keeps (longer groups are read again)
  const int lane = threadIdx.x & (64 * WAVES - 1);
  const int64_t id = WAVES == 4 ? (int64_t)blockIdx.x : (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  const int groups = a.together ? 1 : a.H;
  const int64_t width = a.together ? (int64_t)a.H * a.E : a.E;
  if (id >= a.num_tokens * groups) return;
  const int64_t t = id / groups, at = id % groups * width;
  const float* x = a.work + t * a.wld + at;
  const T* g = (const T*)a.p + t * a.ld + a.g_off + at;
  const T* nw = (const T*)a.norm_w;
  T* o = (T*)a.out + t * a.out_ld + at;
  float v[NR][VEC], ss = 0.f;
  auto read = [&](int64_t e, float (&f)[VEC]) {
    if constexpr (VEC == 4) {
      const float4 q = *reinterpret_cast<const float4*>(x + e);
      f[0] = q.x; f[1] = q.y; f[2] = q.z; f[3] = q.w;
    } else {
      f[0] = x[e];
    }
  };
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int64_t e = (int64_t)i * STEP + lane * VEC;
#pragma unroll
    for (int u = 0; u < VEC; ++u) v[i][u] = 0.f;
    if (e < width) read(e, v[i]);
#pragma unroll
    for (int u = 0; u < VEC; ++u) ss += v[i][u] * v[i][u];
  }
  for (int64_t e = (int64_t)NR * STEP + lane * VEC; e < width; e += STEP) {
    float f[VEC];
    read(e, f);
#pragma unroll
    for (int u = 0; u < VEC; ++u) ss += f[u] * f[u];
  }
  ss = WAVES == 4 ? block_sum(ss, red) : wave_sum(ss);
  const float rs = 1.0f / sqrtf(ss / (float)width + a.eps);
  auto put = [&](int64_t e, const float (&f)[VEC]) {
    T gv[VEC], wv[VEC], r[VEC];
    if constexpr (VEC == 4 && sizeof(T) == 2) {
      *reinterpret_cast<uint2*>(gv) = *reinterpret_cast<const uint2*>(g + e);
      *reinterpret_cast<uint2*>(wv) = *reinterpret_cast<const uint2*>(nw + e);
    } else {
#pragma unroll
      for (int u = 0; u < VEC; ++u) {
        gv[u] = g[e + u];
        wv[u] = nw[e + u];
      }
    }
#pragma unroll
    for (int u = 0; u < VEC; ++u) {
      const float gf = Elem<T>::to_f(gv[u]);
      r[u] = Elem<T>::from_f(f[u] * rs * Elem<T>::to_f(wv[u]) * lin_sigmoid(gf) * (a.gate_silu ? gf : 1.0f));
    }
    if constexpr (VEC == 4 && sizeof(T) == 2)
      *reinterpret_cast<uint2*>(o + e) = *reinterpret_cast<const uint2*>(r);
    else
#pragma unroll
      for (int u = 0; u < VEC; ++u) o[e + u] = r[u];
  };
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int64_t e = (int64_t)i * STEP + lane * VEC;
    if (e < width) put(e, v[i]);
  }
  for (int64_t e = (int64_t)NR * STEP + lane * VEC; e < width; e += STEP) {
    float f[VEC];
    read(e, f);
    put(e, f);
  }
}

}  // namespace semipd

using namespace semipd;

static int64_t linear_row_width(int num_heads, int v_dim) { return ((int64_t)num_heads * v_dim + 3) / 4 * 4; }
static int linear_nd(int qk_dim) { return qk_dim <= 64 ? 2 : (qk_dim <= 128 ? 4 : 8); }
static bool linear_chunk_shape(int qk_dim, int v_dim, int dtype) {
  return dtype == SEMIPD_BF16 && qk_dim % 8 == 0 && qk_dim <= 256 && v_dim % 8 == 0;
}
// as many chunks as the portions can have: a whole one for every 64 tokens and a short one for every request
static int64_t linear_max_chunks(int64_t num_tokens, int64_t batch) { return num_tokens / kLinChunk + batch; }

extern "C" int64_t semipd_linear_attention_workspace(int64_t num_tokens, int64_t batch, int num_heads, int qk_dim, int v_dim, int extend,
                                                     int dtype) {
  const int64_t rows = num_tokens * linear_row_width(num_heads, v_dim);
  if (!extend) return rows;
  if (!linear_chunk_shape(qk_dim, v_dim, dtype)) return rows + num_tokens * num_heads * qk_dim;
  const int nd = linear_nd(qk_dim);
  return rows + linear_max_chunks(num_tokens, batch) * num_heads * ((int64_t)lin_frags(nd) * 256 + 32 * nd);
}

extern "C" int semipd_linear_attention(const void* proj, int64_t ld, int64_t q_off, int64_t k_off, int64_t v_off, int64_t g_off,
                                       int64_t a_off, int rank, const void* a2, const float* a2_bias, float tau, const float* powers,
                                       int qkv_silu, const void* norm_w, int norm_together, float eps, int gate_silu, float* work,
                                       int64_t work_elems, float* state, int64_t state_ld, const int64_t* state_indices,
                                       const int64_t* seq_lens, const int32_t* q_start, const int32_t* q_len, int64_t batch,
                                       int64_t num_tokens, int num_heads, int qk_dim, int v_dim, float q_scale, void* out,
                                       int64_t out_ld, int form, int dtype, void* stream) {
  SEMIPD_CHECK_ARG(batch >= 0 && num_tokens >= 0, SEMIPD_EINVAL, "linear_attention: bad sizes");
  if (batch == 0 || num_tokens == 0) return 0;
  SEMIPD_CHECK_ARG(num_heads > 0 && qk_dim > 0 && v_dim > 0 && qk_dim <= 1024, SEMIPD_ESHAPE,
                   "linear_attention: %d heads of %d x %d (keys of at most 1024 elements)", num_heads, qk_dim, v_dim);
  SEMIPD_CHECK_ARG(proj && norm_w && work && state && state_indices && seq_lens && out, SEMIPD_EINVAL, "linear_attention: null pointer");
  SEMIPD_CHECK_ARG((a2 != nullptr) != (powers != nullptr), SEMIPD_EINVAL, "linear_attention: a decay per channel or one per head");
  SEMIPD_CHECK_ARG(!a2 || (a2_bias && rank > 0 && tau > 0.f), SEMIPD_EINVAL, "linear_attention: a per-channel decay of rank %d", rank);
  SEMIPD_CHECK_ARG((q_start == nullptr) == (q_len == nullptr), SEMIPD_EINVAL, "linear_attention: q_start and q_len come together");
  SEMIPD_CHECK_ARG(q_start != nullptr || num_tokens == batch, SEMIPD_EINVAL, "linear_attention: one row per request without q_start");
  const int64_t qk = (int64_t)num_heads * qk_dim, vv = (int64_t)num_heads * v_dim;
  SEMIPD_CHECK_ARG(q_off >= 0 && k_off >= 0 && v_off >= 0 && g_off >= 0 && ld >= q_off + qk && ld >= k_off + qk && ld >= v_off + vv &&
                       ld >= g_off + vv && (!a2 || (a_off >= 0 && ld >= a_off + rank)),
                   SEMIPD_EINVAL, "linear_attention: a column range leaves the row");
  const int64_t work_ld = linear_row_width(num_heads, v_dim);
  SEMIPD_CHECK_ARG(work_elems >= semipd_linear_attention_workspace(num_tokens, batch, num_heads, qk_dim, v_dim, q_start != nullptr, dtype) &&
                       out_ld >= vv && state_ld >= (int64_t)num_heads * qk_dim * v_dim,
                   SEMIPD_EINVAL, "linear_attention: rows too short");
  SEMIPD_CHECK_ARG(batch <= 65535 && num_heads <= 65535, SEMIPD_ESHAPE, "linear_attention: too many requests or heads");
  float* rest = work + num_tokens * work_ld;
  LinArgs a{proj, ld, q_off, k_off, v_off, g_off, a_off, rank, a2, a2_bias, a2 ? 1.0f / tau : 0.f, powers, qkv_silu, work, work_ld,
            rest, nullptr, nullptr, state, state_ld, state_indices, seq_lens, q_start, q_len, batch, num_tokens, num_heads, qk_dim, v_dim,
            q_scale, norm_w, norm_together, eps, gate_silu, out, out_ld};
  hipStream_t s = as_stream(stream);
  if (q_start == nullptr) {
    const bool vec = v_dim % 4 == 0 && state_ld % 4 == 0 && aligned16(state);
    const int cols = vec ? 64 : 16;
    const size_t bytes = ((size_t)(3 * qk_dim + 3) / 4 * 4 + 16 * (size_t)cols) * sizeof(float);
    const dim3 grid((unsigned)((v_dim + cols - 1) / cols), (unsigned)num_heads, (unsigned)batch);
    SEMIPD_DISPATCH_DTYPE(dtype, T, {
      if (vec) hipLaunchKernelGGL((linear_step_kernel<T, 4>), grid, dim3(256), bytes, s, a);
      else hipLaunchKernelGGL((linear_step_kernel<T, 1>), grid, dim3(256), bytes, s, a);
    });
  } else {
    const bool chunk_ok = linear_chunk_shape(qk_dim, v_dim, dtype) && aligned16(proj) && ld % 8 == 0 && q_off % 8 == 0 && k_off % 8 == 0 &&
                          v_off % 8 == 0 && aligned16(work);
    SEMIPD_CHECK_ARG(form != 2 || chunk_ok, SEMIPD_ESHAPE, "linear_attention: the matrix-core form does not take this shape or type");
    if (chunk_ok && form != 1) {
      const int nd = linear_nd(qk_dim);
      const int64_t chunks = linear_max_chunks(num_tokens, batch);
      a.frags = reinterpret_cast<uint8_t*>(rest);
      a.keep = rest + chunks * num_heads * lin_frags(nd) * 256;
      const dim3 pgrid((unsigned)chunks, (unsigned)num_heads);
      // one workgroup fits a CU: 32 columns of S each while they all run at once, 64 otherwise
      const int cus = owned_cus().load() > 0 ? owned_cus().load() : 256;
      const bool wide = batch * num_heads * ((v_dim + 31) / 32) > cus;
      const int64_t items = batch * num_heads * ((v_dim + (wide ? 63 : 31)) / (wide ? 64 : 32));
      const dim3 wgrid((unsigned)((items + 7) / 8 * 8));
      static std::atomic<uint64_t> done[12] = {};
#define SEMIPD_LIN_LAUNCH(K, GRID, THREADS, BYTES, SLOT)                                                                       \
  do {                                                                                                                        \
    constexpr size_t bytes = BYTES;                                                                                           \
    if (bytes > 65536 && ensure_dynamic_lds((const void*)K, bytes, done[SLOT], "linear_attention")) return SEMIPD_EINVAL;     \
    hipLaunchKernelGGL(K, GRID, dim3(THREADS), bytes, s, a);                                                                  \
  } while (0)
#define SEMIPD_LIN_CHUNKS(ND, SLOT)                                                                                            \
  do {                                                                                                                        \
    if (a2) SEMIPD_LIN_LAUNCH((channel_operands_kernel<ND>), pgrid, 256, channel_lds<ND>(), SLOT);                            \
    else SEMIPD_LIN_LAUNCH((head_operands_kernel<ND>), pgrid, 256, 2 * (size_t)kLinChunk * lin_row(ND), SLOT + 1);            \
    if (wide) SEMIPD_LIN_LAUNCH((chunk_walk_kernel<ND, 4>), wgrid, 512, (walk_lds<ND, 4>()), SLOT + 2);                       \
    else SEMIPD_LIN_LAUNCH((chunk_walk_kernel<ND, 2>), wgrid, 512, (walk_lds<ND, 2>()), SLOT + 3);                            \
  } while (0)
      if (nd == 2) SEMIPD_LIN_CHUNKS(2, 0);
      else if (nd == 4) SEMIPD_LIN_CHUNKS(4, 4);
      else SEMIPD_LIN_CHUNKS(8, 8);
#undef SEMIPD_LIN_CHUNKS
#undef SEMIPD_LIN_LAUNCH
    } else {
      if (a2) {
        const dim3 grid((unsigned)((num_tokens * qk + 255) / 256));
        SEMIPD_DISPATCH_DTYPE(dtype, T, hipLaunchKernelGGL((channel_decay_kernel<T>), grid, dim3(256), 0, s, a));
      }
#define SEMIPD_LIN_SCAN(NPT, NS, STAGE)                                                                                        \
  do {                                                                                                                        \
    constexpr int cols = 64 / NS;                                                                                             \
    const unsigned blocks = (unsigned)(batch * num_heads * ((v_dim + cols - 1) / cols));                                      \
    const size_t bytes = (size_t)STAGE * (3 * NPT * NS + cols) * sizeof(float);                                               \
    SEMIPD_DISPATCH_DTYPE(dtype, T,                                                                                           \
                          hipLaunchKernelGGL((linear_scan_kernel<T, NPT, NS>), dim3(blocks), dim3(64), bytes, s, a, STAGE));   \
  } while (0)
      if (qk_dim <= 32) SEMIPD_LIN_SCAN(32, 1, 8);
      else if (qk_dim <= 64) SEMIPD_LIN_SCAN(32, 2, 8);
      else if (qk_dim <= 128) SEMIPD_LIN_SCAN(32, 4, 8);
      else if (qk_dim <= 256) SEMIPD_LIN_SCAN(32, 8, 8);
      else if (qk_dim <= 512) SEMIPD_LIN_SCAN(32, 16, 8);
      else SEMIPD_LIN_SCAN(64, 16, 4);
#undef SEMIPD_LIN_SCAN
    }
  }
  const int64_t esz = dtype == SEMIPD_F32 ? 4 : 2, vb = 4 * esz;
  const bool vec = v_dim % 4 == 0 && aligned16(work) && (uintptr_t)out % vb == 0 && out_ld % 4 == 0 && (uintptr_t)norm_w % vb == 0 &&
                   (uintptr_t)proj % vb == 0 && ld % 4 == 0 && g_off % 4 == 0;
  const int64_t groups = num_tokens * (norm_together ? 1 : num_heads);
  const bool block = (norm_together ? vv : v_dim) > 1024;
  const dim3 ogrid((unsigned)(block ? groups : (groups + 3) / 4));
  SEMIPD_DISPATCH_DTYPE(dtype, T, {
    if (vec && block) hipLaunchKernelGGL((linear_out_kernel<T, 4, 4>), ogrid, dim3(256), 0, s, a);
    else if (vec) hipLaunchKernelGGL((linear_out_kernel<T, 4, 1>), ogrid, dim3(256), 0, s, a);
    else if (block) hipLaunchKernelGGL((linear_out_kernel<T, 1, 4>), ogrid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL((linear_out_kernel<T, 1, 1>), ogrid, dim3(256), 0, s, a);
  });
  return launch_status("linear_attention");
}
