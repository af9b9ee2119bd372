// stack_latent.hip — attention over a latent cache on the matrix cores (vra_stack_attention sends its shared-row form here), gfx950.
//
// The cache holds ONE row [latent | rotated key part] per token: every head's keys are the whole row, its values the row's first columns.
// So the rows a workgroup stages in LDS serve all heads, as keys and as values.  Query rows are (token, head) pairs; a wave owns 16 of
// them and walks the keys in tiles of 32 aligned to absolute positions:
//   S^T = K . Q^T    A operand = key rows (ds_read_b128), B = the wave's query rows, kept in registers;
//   O^T += V^T . P^T  A operand = the same tile read transposed (ds_read_b64_tr_b16), B = the lane's own weights, split into a bf16 head
//                    and a bf16 tail (p = hi + lo to 2^-17), so that the weights stay f32 in effect.
// Tiles come from the paged cache straight into LDS (16 bytes a lane, no registers), one tile ahead of the arithmetic.
//
// One token per sequence (decode): a workgroup takes 16 heads and every S-th tile of 64 keys of a sequence.  Its four waves score 16 keys each,
// exchange maxima and weights through LDS and then own a quarter of the value channels each; a second launch joins the S partial sums, the
// sink and the output gate.  S is fixed for a model, tiles are assigned by absolute position: one order of the sums, graph-capturable.
//
// A prompt row's running reference moves only when a score exceeds it by more than 8 (weights then stay below e^8, sums are f32): a decision of
// the row alone.  Tiles without a visible key change nothing.  So a row's result does not depend on the rows it shares a wave with, on
// the portion its token came in or on the pages.
#include <algorithm>

#include "stack_common.cuh"
#include "stack_launch.h"

namespace {

typedef short s16x4_t __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) s16x4_t* lds_s16x4_ptr;
typedef __attribute__((address_space(3))) void* lds_void_ptr;
typedef __attribute__((address_space(1))) const void* glb_void_ptr;

// A tile in LDS: 32 rows of 4 * DC chunks of 16 bytes, chunk c of row r at place c ^ lat_swz(r): the 16 rows that a fragment read touches at
// one chunk lie in 16 different bank groups, and so do the row groups of a transposed read.
__device__ __forceinline__ int lat_swz(int r) { return (((r >> 1) & 3) << 1) | ((r >> 3) & 1); }

// DC: 32-channel steps of a row (even), VT: 16-channel tiles of the values, NW: waves
template <int DC, int VT, int NW>
__global__ __launch_bounds__(64 * NW) void stk_latent_prefill_kernel(StkAttnArgs a) {
  static_assert(DC % 2 == 0 && VT % 2 == 0, "whole swizzle groups");
  constexpr int KT = 32, RC = 4 * DC, ROWB = RC * 16, TILEB = KT * ROWB, NL = RC / 2;  // NL: 1-KiB loads of a tile
  extern __shared__ __attribute__((aligned(1024))) unsigned char smem[];
  __shared__ long long wmax[NW], wmin[NW];
  const int b = blockIdx.y, H = a.H, dim = a.dim, vdim = a.vdim;
  const int q0 = a.cu_q[b], q1 = a.cu_q[b + 1];
  const int n_rows = (q1 - q0) * H;
  // the last rows of a portion see the most keys: they are dispatched first
  const int r0 = ((int)gridDim.x - 1 - (int)blockIdx.x) * 16 * NW;
  if (r0 >= n_rows) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), rq = lane & 15, oct = lane >> 4;
  const int r = r0 + wave * 16 + rq;
  const bool qv = r < n_rows;
  const int tq = q0 + (qv ? r / H : 0), head = qv ? r % H : 0;
  const int64_t pq = qv ? a.positions[tq] : -1;
  s16x8 qf[DC];
  {
    const uint16_t* q = (const uint16_t*)a.q + (size_t)tq * a.ldq + (size_t)head * dim;
    const u32x4 zero4 = {0u, 0u, 0u, 0u};
#pragma unroll
    for (int c = 0; c < DC; c++) {
      const int ch = c * 32 + oct * 8;
      const bool ok = qv && ch < dim;
      const u32x4 v = *(const u32x4*)(q + (ok ? ch : 0));
      qf[c] = __builtin_bit_cast(s16x8, ok ? v : zero4);
    }
  }
  const float sc = a.scale * (a.head_scale ? a.head_scale[head] : 1.f);
  int64_t key_lo64 = a.window > 0 && pq >= 0 ? max((int64_t)0, pq - a.window + 1) : 0;
  int64_t pmax = pq, lmin = pq >= 0 ? key_lo64 : INT64_MAX;
  for (int o = 32; o > 0; o >>= 1) {
    pmax = max(pmax, (int64_t)__shfl_xor((long long)pmax, o, 64));
    lmin = min(lmin, (int64_t)__shfl_xor((long long)lmin, o, 64));
  }
  if (lane == 0) wmax[wave] = pmax, wmin[wave] = lmin;
  __syncthreads();
  int64_t gmax = wmax[0], gmin = wmin[0];
  for (int w = 1; w < NW; w++) gmax = max(gmax, (int64_t)wmax[w]), gmin = min(gmin, (int64_t)wmin[w]);
  const int kt_begin = gmin == INT64_MAX ? 0 : __builtin_amdgcn_readfirstlane((int)(gmin / KT) * KT);
  const int n_keys = __builtin_amdgcn_readfirstlane((int)min((int64_t)a.context_lens[b], gmax + 1));
  // keys any row of this wave sees
  const int wave_end = __builtin_amdgcn_readfirstlane((int)min((int64_t)n_keys, pmax + 1));
  const int wave_lo = __builtin_amdgcn_readfirstlane(lmin == INT64_MAX ? 0 : (int)lmin);
  const int key_lo = (int)key_lo64, key_end = (int)min((int64_t)n_keys, pq + 1);
  const uint16_t* kc = (const uint16_t*)a.kc;
  const uint32_t* bt = a.block_tables + (size_t)b * a.max_blocks;
  const int k_ld = a.k_ld;
  // one tile -> LDS.  The page size is a multiple of 32: a tile lies in one page.  Rows beyond the last key repeat it (their weights are 0);
  // chunks beyond the row read its first one (the query's channels there are 0).
  auto request_tile = [&](int buf, int kt0) {
    const int64_t slot0 = (int64_t)bt[kt0 / a.BS] * a.BS + kt0 % a.BS;
    const uint16_t* base = kc + slot0 * k_ld;
    const int last = n_keys - 1 - kt0;
#pragma unroll
    for (int k = 0; k < (NL + NW - 1) / NW; k++) {
      const int idx = k * NW + wave;
      if (NL % NW == 0 || idx < NL) {
        const int p = idx * 64 + lane, row = p / RC, c = (p % RC) ^ lat_swz(row);
        const int off = min(row, last) * k_ld + (c * 8 < dim ? c * 8 : 0);
        __builtin_amdgcn_global_load_lds((glb_void_ptr)(base + off), (lds_void_ptr)(smem + buf * TILEB + idx * 1024), 16, 0, 0);
      }
    }
  };
  // LDS addresses of this lane inside a tile (bytes)
  // (a row's first chunk lies at a multiple of eight chunks: the swizzle and the chunk's low bits meet in address bits 4 .. 6, by exclusive or)
  const int ka = rq * ROWB + (oct ^ lat_swz(rq)) * 16;  // key rq, channels oct * 8 ..; key 16 + rq has the same swizzle
  const int vrow = oct * 4 + (rq >> 2);
  const int va = vrow * ROWB + (((rq & 3) >> 1) ^ lat_swz(vrow)) * 16 + (rq & 1) * 8;
  f32x4 acc[VT];
#pragma unroll
  for (int t = 0; t < VT; t++) acc[t] = vra_zero_acc();
  float m = -INFINITY, l = 0.f;
  if (a.sink) m = a.sink[head], l = oct == 0 ? 1.f : 0.f;  // (the four lanes of a row add their sums at the end: the sink counts once)
  if (kt_begin < n_keys) request_tile(0, kt_begin);
  int buf = 0;
  for (int kt0 = kt_begin; kt0 < n_keys; kt0 += KT, buf ^= 1) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // this wave's part of the tile has arrived ...
    __syncthreads();                                  // ... and so has every wave's; nobody reads the other buffer any more
    if (kt0 + KT < n_keys) request_tile(buf ^ 1, kt0 + KT);
    if (kt0 >= wave_end || kt0 + KT <= wave_lo) continue;  // (wave-uniform: nothing of this tile is visible to the wave's rows)
    const unsigned char* tile = smem + buf * TILEB;
    f32x4 s0 = vra_zero_acc(), s1 = vra_zero_acc();
    s16x8 kf[2][2];
    kf[0][0] = *(const s16x8*)(tile + ka);
    kf[0][1] = *(const s16x8*)(tile + ka + 16 * ROWB);
#pragma unroll
    for (int c = 0; c < DC; c++) {
      if (c + 1 < DC) {
        const int ad = (ka ^ (((c + 1) & 1) << 6)) + ((c + 1) >> 1) * 128;
        kf[(c + 1) & 1][0] = *(const s16x8*)(tile + ad);
        kf[(c + 1) & 1][1] = *(const s16x8*)(tile + ad + 16 * ROWB);
      }
      BF16::mfma(s0, kf[c & 1][0], qf[c]);
      BF16::mfma(s1, kf[c & 1][1], qf[c]);
    }
    VRA_MFMA_DRAIN();
    float pv[8];
    float tmax = -INFINITY;
#pragma unroll
    for (int i = 0; i < 8; i++) {
      const int key = kt0 + (i >> 2) * 16 + oct * 4 + (i & 3);
      const float x = (i < 4 ? s0[i & 3] : s1[i & 3]) * sc;
      pv[i] = key < key_end && key >= key_lo ? x : -INFINITY;
      tmax = fmaxf(tmax, pv[i]);
    }
    tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
    const bool move = tmax > m + 8.f;  // (m = -inf: every finite score moves it; a row without a visible key so far: tmax = -inf, no move)
    if (__any(move)) {
      const float corr = move ? (m > -INFINITY ? __expf(m - tmax) : 0.f) : 1.f;
      m = move ? tmax : m;
      l *= corr;
#pragma unroll
      for (int t = 0; t < VT; t++) acc[t][0] *= corr, acc[t][1] *= corr, acc[t][2] *= corr, acc[t][3] *= corr;
    }
    float psum = 0.f;
#pragma unroll
    for (int i = 0; i < 8; i++) {
      pv[i] = pv[i] > -INFINITY ? __expf(pv[i] - m) : 0.f;
      psum += pv[i];
    }
    l += psum;
    u32x4 phi, plo;
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const float a0 = pv[2 * e], a1 = pv[2 * e + 1];
      const uint32_t hi = BF16::pack2(a0, a1);
      phi[e] = hi;
      plo[e] = BF16::pack2(a0 - __uint_as_float(hi << 16), a1 - __uint_as_float(hi & 0xffff0000u));
    }
    auto vread = [&](int t) {
      const unsigned char* p = tile + (va ^ ((t & 3) << 5)) + (t >> 2) * 128;
      const s16x4_t lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_ptr)(p));
      const s16x4_t hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_ptr)(p + 16 * ROWB));
      return __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
    };
    s16x8 vf[2][2];
    vf[0][0] = vread(0), vf[0][1] = vread(1);
#pragma unroll
    for (int t = 0; t < VT; t += 2) {
      const int u = (t >> 1) & 1;
      if (t + 2 < VT) vf[u ^ 1][0] = vread(t + 2), vf[u ^ 1][1] = vread(t + 3);
      BF16::mfma(acc[t], vf[u][0], __builtin_bit_cast(s16x8, phi));
      BF16::mfma(acc[t + 1], vf[u][1], __builtin_bit_cast(s16x8, phi));
      BF16::mfma(acc[t], vf[u][0], __builtin_bit_cast(s16x8, plo));
      BF16::mfma(acc[t + 1], vf[u][1], __builtin_bit_cast(s16x8, plo));
    }
    VRA_MFMA_DRAIN();
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (!qv) return;
  float inv = l > 0.f ? 1.f / l : 0.f;
  if (a.gate) inv *= sigmoidf_(a.gate[(size_t)tq * a.gate_ld + head]);
  uint16_t* out = (uint16_t*)a.out + ((size_t)tq * H + head) * vdim;
#pragma unroll
  for (int t = 0; t < VT; t++) {
    const int c = t * 16 + oct * 4;
    if (c < vdim) {
      uint2 v;
      v.x = BF16::pack2(acc[t][0] * inv, acc[t][1] * inv);
      v.y = BF16::pack2(acc[t][2] * inv, acc[t][3] * inv);
      *(uint2*)(out + c) = v;
    }
  }
}

// part: f32 [B][S][H][vdim] sums weighted by e^(score - m), then f32 [B][S][H][2] (m, sum of the weights)
template <int DC, int VT>
__global__ __launch_bounds__(256) void stk_latent_decode_kernel(StkAttnArgs a, float* part, int S, int nbuf) {
  static_assert(DC % 2 == 0, "whole swizzle groups");
  constexpr int KT = 64, RC = 4 * DC, ROWB = RC * 16, TILEB = KT * ROWB, NL = RC, TW = (VT + 3) / 4, PLD = KT + 8;
  extern __shared__ __attribute__((aligned(1024))) unsigned char smem[];
  __shared__ float wm[4][16], wl[4][16];
  __shared__ __attribute__((aligned(16))) uint16_t p_hi[16 * PLD], p_lo[16 * PLD];
  const int s = blockIdx.x, b = blockIdx.y, H = a.H, dim = a.dim, vdim = a.vdim;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), rq = lane & 15, oct = lane >> 4;
  const int head = blockIdx.z * 16 + rq;
  const bool hv = head < H;
  const int64_t p = a.positions[b];
  const int n_keys = __builtin_amdgcn_readfirstlane((int)min((int64_t)a.context_lens[b], p + 1));
  const int key_lo = __builtin_amdgcn_readfirstlane(a.window > 0 ? (int)max((int64_t)0, p - a.window + 1) : 0);
  float* ml = part + (size_t)gridDim.y * S * H * vdim + (((size_t)b * S + s) * H + head) * 2;
  // this workgroup's first tile: the smallest tile index t >= key_lo / 64 with t mod S = s
  const int t_lo = key_lo / KT;
  int kt0 = (t_lo + (s - t_lo % S + S) % S) * KT;
  if (kt0 >= n_keys) {
    if (wave == 0 && oct == 0 && hv) ml[0] = -INFINITY, ml[1] = 0.f;
    return;
  }
  const uint16_t* kc = (const uint16_t*)a.kc;
  const uint32_t* bt = a.block_tables + (size_t)b * a.max_blocks;
  const int k_ld = a.k_ld;
  auto request_tile = [&](int buf, int k0) {  // (the page size is a multiple of 64: a tile lies in one page)
    const int64_t slot0 = (int64_t)bt[k0 / a.BS] * a.BS + k0 % a.BS;
    const uint16_t* base = kc + slot0 * k_ld;
    const int last = n_keys - 1 - k0;
#pragma unroll
    for (int k = 0; k < NL / 4; k++) {
      const int idx = k * 4 + wave;
      const int pl = idx * 64 + lane, row = pl / RC, c = (pl % RC) ^ lat_swz(row);
      const int off = min(row, last) * k_ld + (c * 8 < dim ? c * 8 : 0);
      __builtin_amdgcn_global_load_lds((glb_void_ptr)(base + off), (lds_void_ptr)(smem + buf * TILEB + idx * 1024), 16, 0, 0);
    }
  };
  request_tile(0, kt0);
  s16x8 qf[DC];
  {
    const uint16_t* q = (const uint16_t*)a.q + (size_t)b * a.ldq + (size_t)(hv ? head : 0) * dim;
    const u32x4 zero4 = {0u, 0u, 0u, 0u};
#pragma unroll
    for (int c = 0; c < DC; c++) {
      const int ch = c * 32 + oct * 8;
      const bool ok = hv && ch < dim;
      const u32x4 v = *(const u32x4*)(q + (ok ? ch : 0));
      qf[c] = __builtin_bit_cast(s16x8, ok ? v : zero4);
    }
  }
  const float sc = a.scale * (a.head_scale && hv ? a.head_scale[head] : 1.f);
  const int ka = (wave * 16 + rq) * ROWB + (oct ^ lat_swz(rq)) * 16;
  const int vrow = oct * 4 + (rq >> 2);
  const int va = vrow * ROWB + (((rq & 3) >> 1) ^ lat_swz(vrow)) * 16 + (rq & 1) * 8;
  f32x4 acc[TW];
#pragma unroll
  for (int t = 0; t < TW; t++) acc[t] = vra_zero_acc();
  float m = -INFINITY, l = 0.f;
  int buf = 0;
  for (; kt0 < n_keys; kt0 += S * KT) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (nbuf == 2 && kt0 + S * KT < n_keys) request_tile(buf ^ 1, kt0 + S * KT);
    const unsigned char* tile = smem + buf * TILEB;
    f32x4 s0 = vra_zero_acc(), s1 = vra_zero_acc();
    s16x8 kf[2][2];
    kf[0][0] = *(const s16x8*)(tile + ka);
    kf[0][1] = *(const s16x8*)(tile + (ka ^ 64));
#pragma unroll
    for (int c = 0; c < DC; c += 2) {
      const int u = (c >> 1) & 1;
      if (c + 2 < DC) {
        kf[u ^ 1][0] = *(const s16x8*)(tile + ka + ((c + 2) >> 1) * 128);
        kf[u ^ 1][1] = *(const s16x8*)(tile + (ka ^ 64) + ((c + 2) >> 1) * 128);
      }
      BF16::mfma(s0, kf[u][0], qf[c]);
      BF16::mfma(s1, kf[u][1], qf[c + 1]);
    }
    VRA_MFMA_DRAIN();
    float pv[4], tmax = -INFINITY;
#pragma unroll
    for (int j = 0; j < 4; j++) {
      const int key = kt0 + wave * 16 + oct * 4 + j;
      const float x = (s0[j] + s1[j]) * sc;
      pv[j] = key < n_keys && key >= key_lo ? x : -INFINITY;
      tmax = fmaxf(tmax, pv[j]);
    }
    tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
    if (oct == 0) wm[wave][rq] = tmax;
    __syncthreads();
    // (the tile holds at least one visible key: the maximum is finite)
    const float mn = fmaxf(m, fmaxf(fmaxf(wm[0][rq], wm[1][rq]), fmaxf(wm[2][rq], wm[3][rq])));
    const float corr = m > -INFINITY ? __expf(m - mn) : 0.f;
    m = mn;
    float psum = 0.f;
#pragma unroll
    for (int j = 0; j < 4; j++) {
      pv[j] = pv[j] > -INFINITY ? __expf(pv[j] - mn) : 0.f;
      psum += pv[j];
    }
    l = l * corr + psum;
    {
      uint2 hi, lo;
      hi.x = BF16::pack2(pv[0], pv[1]), hi.y = BF16::pack2(pv[2], pv[3]);
      lo.x = BF16::pack2(pv[0] - __uint_as_float(hi.x << 16), pv[1] - __uint_as_float(hi.x & 0xffff0000u));
      lo.y = BF16::pack2(pv[2] - __uint_as_float(hi.y << 16), pv[3] - __uint_as_float(hi.y & 0xffff0000u));
      const int at = rq * PLD + (wave >> 1) * 32 + oct * 8 + (wave & 1) * 4;  // keys in the order of a transposed read's halves
      *(uint2*)(p_hi + at) = hi;
      *(uint2*)(p_lo + at) = lo;
    }
    __syncthreads();
#pragma unroll
    for (int t = 0; t < TW; t++) acc[t][0] *= corr, acc[t][1] *= corr, acc[t][2] *= corr, acc[t][3] *= corr;
    s16x8 pf[2][2];
#pragma unroll
    for (int ks = 0; ks < 2; ks++) {
      pf[ks][0] = *(const s16x8*)(p_hi + rq * PLD + ks * 32 + oct * 8);
      pf[ks][1] = *(const s16x8*)(p_lo + rq * PLD + ks * 32 + oct * 8);
    }
    // value tiles wave, wave + 4, ..: their places in a row differ by whole swizzle groups
    const unsigned char* vp = tile + (va ^ (wave << 5));
    s16x8 vf[TW][2];
#pragma unroll
    for (int t = 0; t < TW; t++)
#pragma unroll
      for (int ks = 0; ks < 2; ks++) {
        const unsigned char* q = vp + t * 128 + ks * 32 * ROWB;
        const s16x4_t lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_ptr)(q));
        const s16x4_t hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_ptr)(q + 16 * ROWB));
        vf[t][ks] = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
      }
#pragma unroll
    for (int ks = 0; ks < 2; ks++)
#pragma unroll
      for (int e = 0; e < 2; e++)
#pragma unroll
        for (int t = 0; t < TW; t++) BF16::mfma(acc[t], vf[t][ks], pf[ks][e]);
    VRA_MFMA_DRAIN();
    if (nbuf == 1 && kt0 + S * KT < n_keys) {
      __syncthreads();  // (everyone has read the tile)
      request_tile(0, kt0 + S * KT);
    }
    if (nbuf == 2) buf ^= 1;
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (oct == 0) wl[wave][rq] = l;
  __syncthreads();
  if (!hv) return;
  if (wave == 0 && oct == 0) ml[0] = m, ml[1] = (wl[0][rq] + wl[1][rq]) + (wl[2][rq] + wl[3][rq]);
  float* o = part + (((size_t)b * S + s) * H + head) * vdim;
#pragma unroll
  for (int t = 0; t < TW; t++) {
    const int c = (wave + 4 * t) * 16 + oct * 4;
    if (c < vdim) *(float4*)(o + c) = make_float4(acc[t][0], acc[t][1], acc[t][2], acc[t][3]);
  }
}

// joins the S parts of a (sequence, head): out = sum_s e^(m_s - M) o_s / (sum_s e^(m_s - M) l_s + e^(sink - M)) * sigmoid(gate); S <= 64
__global__ __launch_bounds__(128) void stk_latent_decode_join_kernel(StkAttnArgs a, const float* part, int S) {
  __shared__ float ws[64];
  __shared__ float total;
  const int b = blockIdx.x, h = blockIdx.y, H = a.H, vdim = a.vdim, tid = threadIdx.x;
  const float* ml = part + (size_t)gridDim.x * S * H * vdim;
  if (tid < 64) {
    const size_t at = (((size_t)b * S + (tid < S ? tid : 0)) * H + h) * 2;
    const float ms = tid < S ? ml[at] : -INFINITY, ls = tid < S ? ml[at + 1] : 0.f;
    const float sink = a.sink ? a.sink[h] : -INFINITY;
    const float M = fmaxf(wave_max(ms), sink);
    const float w = ms > -INFINITY ? __expf(ms - M) : 0.f;
    ws[tid] = w;
    const float L = wave_sum(w * ls) + (a.sink ? __expf(sink - M) : 0.f);
    if (tid == 0) total = L > 0.f ? (a.gate ? sigmoidf_(a.gate[(size_t)b * a.gate_ld + h]) : 1.f) / L : 0.f;
  }
  __syncthreads();
  const float inv = total;
  uint16_t* out = (uint16_t*)a.out + ((size_t)b * H + h) * vdim;
  for (int c = tid * 4; c < vdim; c += 512) {
    float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
    // eight parts' rows are requested together; a part without a key has weight 0 and an unwritten row: not read
    for (int s0 = 0; s0 < S; s0 += 8) {
      float4 v[8];
#pragma unroll
      for (int u = 0; u < 8; u++) {
        const int s = s0 + u;
        const bool in = s < S && ws[s < S ? s : 0] > 0.f;
        v[u] = in ? *(const float4*)(part + (((size_t)b * S + s) * H + h) * vdim + c) : make_float4(0.f, 0.f, 0.f, 0.f);
      }
#pragma unroll
      for (int u = 0; u < 8; u++) {
        const float w = s0 + u < S ? ws[s0 + u] : 0.f;
        o.x = fmaf(w, v[u].x, o.x), o.y = fmaf(w, v[u].y, o.y), o.z = fmaf(w, v[u].z, o.z), o.w = fmaf(w, v[u].w, o.w);
      }
    }
    uint2 r;
    r.x = BF16::pack2(o.x * inv, o.y * inv), r.y = BF16::pack2(o.z * inv, o.w * inv);
    *(uint2*)(out + c) = r;
  }
}

// the shapes both forms take
bool latent_shape(const StkAttnArgs& a, int dtype) {
  return dtype == VRA_BF16 && a.G == 1 && a.kc == a.vc && a.k_ld == a.v_ld && a.k_ld >= a.dim && a.dim % 8 == 0 && a.vdim % 16 == 0 && a.dim <= 576 &&
         a.vdim <= 512 && a.vdim <= a.dim && a.ldq % 8 == 0 && a.k_ld % 8 == 0 && (uintptr_t)a.q % 16 == 0 && (uintptr_t)a.kc % 16 == 0 &&
         (uintptr_t)a.out % 16 == 0 && a.softcap <= 0.f && a.temp_every <= 0 && a.chunk <= 0;
}

}  // namespace

// tiles of 64 keys a query may see, at most 32 parts (longer ranges: several tiles a part), and no more than the scratch memory allows
int vra_stack_latent_splits(int window, int max_len, int max_seqs, int heads, int vdim) {
  const int64_t keys = window > 0 ? std::min<int64_t>(window + 63, std::max(max_len, 1)) : std::max(max_len, 1);
  int64_t s = std::min<int64_t>(32, std::max<int64_t>(1, (keys + 63) / 64));
  while (s > 1 && (int64_t)max_seqs * s * heads * (vdim + 2) * 4 > (int64_t)512 << 20) s--;
  return (int)s;
}

bool vra_stack_latent_decode(const StkAttnArgs& a, int dtype, int64_t stream) {
  if (!latent_shape(a, dtype) || a.cu_q || !a.scratch || a.splits < 1 || a.splits > 64 || a.BS % 64 != 0 || a.B > 65535) return false;
  if ((size_t)a.B * a.splits * a.H * (a.vdim + 2) * sizeof(float) > a.scratch_bytes) return false;
  hipStream_t st = as_stream(stream);
  const dim3 grid(a.splits, a.B, (a.H + 15) / 16);
  // one tile a part when the splits cover the window: no second buffer
  const int nbuf = a.window > 0 && (a.window + 63 + 63) / 64 <= a.splits ? 1 : 2;
#define STK_LATD(DCV, VTV)                                                                                                                        \
  do {                                                                                                                                            \
    const size_t lds = (size_t)nbuf * 64 * (4 * DCV) * 16;                                                                                        \
    static bool attr = false;                                                                                                                     \
    if (!attr) {                                                                                                                                  \
      (void)hipFuncSetAttribute((const void*)stk_latent_decode_kernel<DCV, VTV>, hipFuncAttributeMaxDynamicSharedMemorySize, 152 * 1024);          \
      attr = true;                                                                                                                                \
    }                                                                                                                                             \
    launch_checked("stack latent attention (decode)", [&] { stk_latent_decode_kernel<DCV, VTV><<<grid, 256, lds, st>>>(a, a.scratch, a.splits, nbuf); }); \
  } while (0)
  if (a.dim <= 128 && a.vdim <= 128) STK_LATD(4, 8);
  else if (a.dim <= 192) STK_LATD(6, 12);
  else if (a.dim <= 256) STK_LATD(8, 16);
  else if (a.dim <= 384) STK_LATD(12, 24);
  else STK_LATD(18, 32);
#undef STK_LATD
  launch_checked("stack latent attention (join)", [&] { stk_latent_decode_join_kernel<<<dim3(a.B, a.H), 128, 0, st>>>(a, a.scratch, a.splits); });
  return true;
}

bool vra_stack_latent_prefill(const StkAttnArgs& a, int dtype, int64_t stream) {
  if (!latent_shape(a, dtype) || !a.cu_q || a.BS % 32 != 0) return false;
  hipStream_t st = as_stream(stream);
  // enough rows for 128 of them on every CU: eight waves share a tile; fewer: four
  const int nw = (int64_t)a.T * a.H >= 256 * 128 ? 8 : 4;
  const dim3 grid((unsigned)(((int64_t)a.max_q * a.H + 16 * nw - 1) / (16 * nw)), a.B);
#define STK_LAT(DCV, VTV, NWV)                                                                                                                    \
  do {                                                                                                                                            \
    const size_t lds = 2 * 32 * (size_t)(4 * DCV) * 16;                                                                                           \
    static bool attr = false;                                                                                                                     \
    if (!attr) {                                                                                                                                  \
      (void)hipFuncSetAttribute((const void*)stk_latent_prefill_kernel<DCV, VTV, NWV>, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);    \
      attr = true;                                                                                                                                \
    }                                                                                                                                             \
    launch_checked("stack latent attention (prefill)", [&] { stk_latent_prefill_kernel<DCV, VTV, NWV><<<grid, 64 * NWV, lds, st>>>(a); });        \
  } while (0)
#define STK_LATW(DCV, VTV)            \
  do {                                \
    if (nw == 8) STK_LAT(DCV, VTV, 8); \
    else STK_LAT(DCV, VTV, 4);        \
  } while (0)
  if (a.dim <= 128 && a.vdim <= 96) STK_LATW(4, 6);
  else if (a.dim <= 192 && a.vdim <= 160) STK_LATW(6, 10);
  else if (a.dim <= 256 && a.vdim <= 192) STK_LATW(8, 12);
  else if (a.dim <= 256) STK_LATW(8, 16);
  else if (a.dim <= 384 && a.vdim <= 384) STK_LATW(12, 24);
  else STK_LATW(18, 32);
#undef STK_LATW
#undef STK_LAT
  return true;
}

// softmax attention over latent rows (keys: whole rows of k_ld elements, values: their first vdim columns) with window, sink, scale and output
// gate per head; scratch (may be null) and splits: the decode form in parts
extern "C" void vra_stack_op_attention_latent(const void* q, int32_t ldq, void* out, const void* cache, int32_t k_ld, const int64_t* positions,
                                              const uint32_t* block_tables, const uint32_t* context_lens, const uint32_t* cu_q, int32_t B, int32_t T,
                                              int32_t max_q, int32_t H, int32_t dim, int32_t vdim, int32_t BS, int32_t max_blocks, float scale, int32_t window,
                                              const float* sink, const float* head_scale, const float* gate, int32_t gate_ld, float* scratch,
                                              int64_t scratch_bytes, int32_t splits, int32_t dtype, int64_t stream) {
  StkAttnArgs a;
  a.q = q, a.ldq = ldq, a.out = out, a.kc = cache, a.vc = cache, a.k_ld = k_ld, a.v_ld = k_ld, a.positions = positions, a.block_tables = block_tables;
  a.context_lens = context_lens, a.cu_q = cu_q, a.B = B, a.T = T, a.max_q = max_q, a.H = H, a.G = 1, a.dim = dim, a.vdim = vdim, a.BS = BS;
  a.max_blocks = max_blocks, a.scale = scale, a.window = window, a.sink = sink, a.head_scale = head_scale, a.gate = gate, a.gate_ld = gate_ld;
  a.scratch = scratch, a.scratch_bytes = (size_t)scratch_bytes, a.splits = splits;
  vra_stack_attention(a, dtype, stream);
}
