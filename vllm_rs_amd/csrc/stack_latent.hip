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
// A row's running reference moves only when a score exceeds it by more than 8 (weights then stay below e^8, sums are f32): a decision of
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

}  // namespace

bool vra_stack_latent_prefill(const StkAttnArgs& a, int dtype, int64_t stream) {
  if (!(dtype == VRA_BF16 && a.cu_q && a.G == 1 && a.kc == a.vc && a.k_ld == a.v_ld && a.k_ld >= a.dim && a.dim % 8 == 0 && a.vdim % 16 == 0 && a.dim <= 576 &&
        a.vdim <= 512 && a.vdim <= a.dim && a.ldq % 8 == 0 && a.k_ld % 8 == 0 && a.BS % 32 == 0 && (uintptr_t)a.q % 16 == 0 && (uintptr_t)a.kc % 16 == 0 &&
        (uintptr_t)a.out % 16 == 0 && a.softcap <= 0.f && a.temp_every <= 0 && a.chunk <= 0))
    return false;
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
