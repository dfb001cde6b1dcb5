// The matrix-core kernel of prompt portions for softmax attention whose queries see a span of the keys, shared by the mixers
// with a paged cache of keys and values and by the one that makes keys and values from latent rows.
#pragma once
#include "common.h"

constexpr float kLog2e = 1.4426950408889634f;

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }

// =============================================================================================
// Prompt portions on the matrix cores (bfloat16 operands, float32 accumulation and softmax).
//
// Grid (query tiles * heads), tile-major, 256 threads.  A tile is up to 128 consecutive tokens of one
// request (int4: request row, first token row, rows, first position); wave w owns rows 32w..32w+31.
// The keys the tile may see are walked 64 at a time, first the kept first keys (when they lie before
// the window of the tile's first row), then the window up to the tile's last row.  A step's keys and
// values come through LDS as padded rows; the next step's are on their way into registers meanwhile.
// Scores are computed transposed, S^T = K Q^T, with v_mfma_f32_32x32x16_bf16: a lane then holds 32
// keys of ONE query, the running softmax needs one cross-lane step, and the probabilities are
// already laid out as the B operand of O^T = V^T P^T.  The V^T operand is read with
// ds_read_b64_tr_b16, which transposes 16-bit elements across the 16 lanes of a group on the way out
// of LDS.  Operand layout (lane l, h = l/32): A[i = l%32][k = 8h..8h+7], B[k = 8h..8h+7][j = l%32],
// D[i = 8(r/4) + 4h + r%4][j = l%32] for the 16 accumulators r.
//
// A key outside the run a step walks is replaced by the nearest one inside when it is loaded (its
// page may have been given back, or not be written yet) and its score is masked.
//
// MODE says where keys and values lie and whether the template's sizes are exact:
//   kSpanPaged   paged cache, key size DK, value size DV,
//   kSpanPadded  paged cache, sizes dk <= DK and dv <= DV (multiples of 8); the rest of a row in LDS is zero,
//   kSpanLatent  one request's keys and values made from its latent rows, in two matrices: row key - key0 of `kcache` holds
//                every head's unrotated key part (dk - e_rot entries at head * (dk - e_rot)) and, from v_off on, every head's
//                value; row key - key0 of `krot` the rotated part (e_rot entries) that the heads share.  The tiles are
//                the portion's own, the last one first; z.portion = (.., first token row, tokens, first position).
// =============================================================================================
typedef __bf16 sp_bf16x8 __attribute__((ext_vector_type(8)));
typedef float sp_v16f __attribute__((ext_vector_type(16)));
typedef float sp_v8f __attribute__((ext_vector_type(8)));
typedef short sp_v4s __attribute__((ext_vector_type(4)));
typedef unsigned sp_v4u __attribute__((ext_vector_type(4)));

constexpr int kSpRows = 128;      // query rows per block
constexpr int kSpKeys = 64;       // keys per step
constexpr int kSpUnits = 256;     // compute units of the chip

enum { kSpanPaged = 0, kSpanPadded = 1, kSpanLatent = 2 };

// What the modes beyond kSpanPaged read besides.
struct SpanSizes {
    int dk, dv;                    // true sizes
    int e_rot, kv_stride, v_off, key0, krot_stride;
    const uint16_t* krot;
    int4 portion;                  // kSpanLatent: (0, first token row, tokens, first position)
};

template <int DK, int DV, int MODE>
__global__ void __launch_bounds__(256, 2)
attn_span_prefill_kernel(const uint16_t* __restrict__ q, int q_stride, uint16_t* __restrict__ out, int out_stride,
                         const uint16_t* __restrict__ gate, int gate_stride,
                         const uint16_t* __restrict__ kcache, const uint16_t* __restrict__ vcache,
                         const int* __restrict__ block_tables, int bt_stride, const int4* __restrict__ tiles,
                         int nh, int nkvh, int page_shift, float scale_log2e, int window, int keep_first, int sink,
                         const float* __restrict__ sinks, float cap_in, const float* __restrict__ slopes, SpanSizes z) {
    // cap_in > 0: a raw score s becomes tanh(s * cap_in) (cap_in = scale / cap) and scale_log2e holds cap * log2 e
    constexpr int NC = DK / 16;           // 16-wide chunks of the key size
    constexpr int ND = DV / 32;           // 32-row tiles of O^T
    constexpr int PK = DK + 8;            // padded row pitches in LDS (elements)
    constexpr int PV = DV + 8;
    constexpr int KCH = DK / 8, VCH = DV / 8;              // 16-byte chunks of a row
    constexpr int LPR = (KCH % 8 == 0 && VCH % 8 == 0) ? 8 : 4;             // threads that fetch a row
    constexpr int RP = 256 / LPR, NP = kSpKeys / RP;                        // rows fetched side by side, passes over a step's rows
    constexpr int NKC = KCH / LPR, NVC = VCH / LPR, NLK = NP * NKC, NLV = NP * NVC;     // loads per row, per thread and step
    static_assert(DK % 32 == 0 && DV % 32 == 0, "a step's rows split evenly over the block");
    // long rows keep one stage in LDS, so that two blocks fit a compute unit
    constexpr bool ONE_STAGE = 2 * kSpKeys * (PK + PV) * 2 > 80 * 1024;
    const int dk = MODE == kSpanPaged ? DK : z.dk, dv = MODE == kSpanPaged ? DV : z.dv, d_plain = dk - z.e_rot;

    // two stages: a step is computed from one while the next step's rows are written into the other (one barrier a step)
    __shared__ __attribute__((aligned(16))) uint16_t Ks0[kSpKeys * PK];
    __shared__ __attribute__((aligned(16))) uint16_t Vs0[kSpKeys * PV];
    __shared__ __attribute__((aligned(16))) uint16_t Ks1[ONE_STAGE ? 8 : kSpKeys * PK];
    __shared__ __attribute__((aligned(16))) uint16_t Vs1[ONE_STAGE ? 8 : kSpKeys * PV];

    const int slot = (int)blockIdx.x;
    const int h = slot % nh;
    // Tiles come longest first.  Where two blocks a unit hold the whole grid, its second half is taken shortest first, so that a
    // unit's two blocks add up to about the same number of steps everywhere.
    const int n_tiles = (int)gridDim.x / nh;
    int place = slot / nh;
    if ((int)gridDim.x <= 2 * kSpUnits && place >= (n_tiles + 1) / 2) place = n_tiles - 1 - (place - (n_tiles + 1) / 2);
    int4 tile;
    if (MODE == kSpanLatent) {
        const int i = (n_tiles - 1 - place) * kSpRows;
        tile = int4{0, z.portion.y + i, z.portion.z - i < kSpRows ? z.portion.z - i : kSpRows, z.portion.w + i};
    } else {
        tile = tiles[place];
    }
    const int req = tile.x, row0 = tile.y, n_rows = tile.z, pos0 = tile.w;
    const int kvh = h / (nh / nkvh);
    const int* bt = MODE == kSpanLatent ? nullptr : block_tables + (size_t)req * bt_stride;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int lq = lane & 31, half = lane >> 5;
    const int page_size = 1 << page_shift, page_mask = page_size - 1;      // pages are a power of two here

    const int my_row = 32 * wave + lq;
    const bool row_ok = my_row < n_rows;
    const int qpos = pos0 + my_row;
    const bool wave_ok = 32 * wave < n_rows;
    const int wave_first = pos0 + 32 * wave;
    const int wave_last = pos0 + ((32 * wave + 31 < n_rows - 1) ? 32 * wave + 31 : n_rows - 1);
    const int last_key = pos0 + n_rows - 1;
    int first_key = (window > 0 && pos0 - window + 1 > 0) ? pos0 - window + 1 : 0;
    int n_kept = keep_first;                           // keys 0 .. n_kept-1 are walked as a run of their own
    if (window == 0 || n_kept >= first_key) { n_kept = 0; if (keep_first >= first_key) first_key = 0; }
    const int kept_steps = (n_kept + kSpKeys - 1) / kSpKeys;
    const int win_kb0 = (first_key / kSpKeys) * kSpKeys;
    const int n_steps = kept_steps + (last_key - win_kb0) / kSpKeys + 1;

    // step -> (first key of the 64, the run's first and last key)
    auto step_of = [&](int s, int& kb, int& klo, int& khi) {
        if (s < kept_steps) { kb = s * kSpKeys; klo = 0; khi = n_kept - 1; }
        else { kb = win_kb0 + (s - kept_steps) * kSpKeys; klo = first_key; khi = last_key; }
    };

    sp_bf16x8 qf[NC];
    {
        const uint16_t* qp = q + (size_t)(row0 + (row_ok ? my_row : 0)) * q_stride + (size_t)h * dk + 8 * half;
#pragma unroll
        for (int c = 0; c < NC; ++c) {                     // rows beyond the tile read row 0 and are never written
            sp_v4u v = {0u, 0u, 0u, 0u};
            if (MODE == kSpanPaged || 16 * c + 8 * half < dk) v = *reinterpret_cast<const sp_v4u*>(qp + 16 * c);
            qf[c] = __builtin_bit_cast(sp_bf16x8, v);
        }
    }
    sp_v16f oacc[ND];
#pragma unroll
    for (int i = 0; i < ND; ++i)
#pragma unroll
        for (int r = 0; r < 16; ++r) oacc[i][r] = 0.f;
    float m = -INFINITY, l = 0.f;

    const size_t khead = (size_t)kvh * page_size * dk, vhead = (size_t)kvh * page_size * dv;
    sp_v4u kreg0[NLK], vreg0[NLV], kreg1[NLK], vreg1[NLV];     // two steps' keys and values on their way: a load has two steps' time to arrive
    // A thread fetches the same rows' pieces of keys and of values, and looks their page ids up a step ahead of the fetch, so a
    // step waits for one trip to memory, not for two in a row.
    const int my_key = tid / LPR, piece = tid % LPR;
    const int k_last = dk / 8 - 1, v_last = dv / 8 - 1;       // (MODE kSpanPaged: never reached beyond)
    const bool padded = MODE != kSpanPaged && (dk < DK || dv < DV);
    int page[NP];
    auto key_of = [&](int s, int kk) -> int {
        int kb, klo, khi;
        step_of(s, kb, klo, khi);
        int key = kb + kk;
        key = key < klo ? klo : key;
        return key > khi ? khi : key;
    };
    auto lookup = [&](int s) {
        if (MODE == kSpanLatent) return;
#pragma unroll
        for (int p = 0; p < NP; ++p) page[p] = bt[key_of(s, my_key + RP * p) >> page_shift];
    };
    auto fetch = [&](int s, sp_v4u* kreg, sp_v4u* vreg) {
#pragma unroll
        for (int p = 0; p < NP; ++p) {
            const int key = key_of(s, my_key + RP * p);
            const uint16_t *kp, *vp, *rp = nullptr;
            if (MODE == kSpanLatent) {
                const uint16_t* row = kcache + (size_t)(key - z.key0) * z.kv_stride;
                kp = row + kvh * d_plain;
                vp = row + z.v_off + kvh * dv;
                rp = z.krot + (size_t)(key - z.key0) * z.krot_stride - d_plain;
            } else {
                const size_t rowi = (((size_t)page[p] * nkvh) << page_shift) + (key & page_mask);
                kp = kcache + khead + rowi * dk;
                vp = vcache + vhead + rowi * dv;
            }
#pragma unroll
            for (int i = 0; i < NKC; ++i) {
                int c = piece + LPR * i;
                if (MODE != kSpanPaged) c = c < k_last ? c : k_last;         // pieces beyond the true size: a real one, cleared on the way to LDS
                const uint16_t* src = (MODE == kSpanLatent && c * 8 >= d_plain) ? rp : kp;
                kreg[p * NKC + i] = *reinterpret_cast<const sp_v4u*>(src + c * 8);
            }
#pragma unroll
            for (int i = 0; i < NVC; ++i) {
                int c = piece + LPR * i;
                if (MODE != kSpanPaged) c = c < v_last ? c : v_last;
                vreg[p * NVC + i] = *reinterpret_cast<const sp_v4u*>(vp + c * 8);
            }
        }
    };
    auto stash = [&](sp_v4u* kreg, sp_v4u* vreg, uint16_t* Ks, uint16_t* Vs) {
        if (padded) {
#pragma unroll
            for (int p = 0; p < NP; ++p) {
#pragma unroll
                for (int i = 0; i < NKC; ++i) if (piece + LPR * i > k_last) kreg[p * NKC + i] = sp_v4u{0u, 0u, 0u, 0u};
#pragma unroll
                for (int i = 0; i < NVC; ++i) if (piece + LPR * i > v_last) vreg[p * NVC + i] = sp_v4u{0u, 0u, 0u, 0u};
            }
        }
#pragma unroll
        for (int p = 0; p < NP; ++p) {
#pragma unroll
            for (int i = 0; i < NKC; ++i) *reinterpret_cast<sp_v4u*>(Ks + (my_key + RP * p) * PK + (piece + LPR * i) * 8) = kreg[p * NKC + i];
#pragma unroll
            for (int i = 0; i < NVC; ++i) *reinterpret_cast<sp_v4u*>(Vs + (my_key + RP * p) * PV + (piece + LPR * i) * 8) = vreg[p * NVC + i];
        }
    };

    // where this lane reads V^T: rows 4 half + (l % 16) / 4 of a 16-key chunk (and 8 rows on), dims 32 dt + 16 (l / 16 % 2) + 4 (l % 4) ..+3
    const int vrow = 4 * half + ((lane & 15) >> 2);
    const int vcol = 16 * ((lane >> 4) & 1) + 4 * (lane & 3);

    // Step s is fetched into registers three steps ahead and written to LDS one step ahead; its page ids are looked up a step before the fetch.
    // (One stage: fetched one step ahead, written between two barriers.)
    lookup(0);
    fetch(0, kreg0, vreg0);
    if (!ONE_STAGE) {
        if (n_steps > 1) { lookup(1); fetch(1, kreg1, vreg1); }
        stash(kreg0, vreg0, Ks0, Vs0);
        if (n_steps > 2) { lookup(2); fetch(2, kreg0, vreg0); }
        if (n_steps > 3) lookup(3);
    } else if (n_steps > 1) {
        lookup(1);
    }
    const float slope = slopes ? slopes[h] * (kLog2e / scale_log2e) : 0.f;      // per token of distance, in units of the scores below
    auto compute = [&](int s, const uint16_t* Ks, const uint16_t* Vs) {
        int kb, klo, khi;
        step_of(s, kb, klo, khi);
        if (!wave_ok || kb > wave_last) return;            // nothing this wave may see
        const bool kept_run = s < kept_steps;
        if (!kept_run && window > 0 && kb + kSpKeys - 1 < wave_first - window + 1 && kb >= keep_first) return;   // all before this wave's windows, none kept

        // ---- S^T = K Q^T : two tiles of 32 keys ----------------------------------
        sp_v16f sacc[2];
#pragma unroll
        for (int tt = 0; tt < 2; ++tt) {
#pragma unroll
            for (int r = 0; r < 16; ++r) sacc[tt][r] = 0.f;
#pragma unroll
            for (int c = 0; c < NC; ++c) {
                const sp_bf16x8 a = *reinterpret_cast<const sp_bf16x8*>(Ks + (32 * tt + lq) * PK + 16 * c + 8 * half);
                sacc[tt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, qf[c], sacc[tt], 0, 0, 0);
            }
        }
        if (cap_in > 0.f) {                                // tanh(z) = 1 - 2 / (1 + e^(2z)): finite for every z
#pragma unroll
            for (int tt = 0; tt < 2; ++tt)
#pragma unroll
                for (int r = 0; r < 16; ++r) {
                    const float e = __builtin_amdgcn_exp2f(sacc[tt][r] * (2.f * kLog2e * cap_in));
                    sacc[tt][r] = 1.f - 2.f * __builtin_amdgcn_rcpf(1.f + e);
                }
        }
        if (slope != 0.f) {
#pragma unroll
            for (int tt = 0; tt < 2; ++tt)
#pragma unroll
                for (int r = 0; r < 16; ++r) sacc[tt][r] -= slope * (float)(qpos - (kb + 32 * tt + 8 * (r >> 2) + 4 * half + (r & 3)));
        }
        // ---- mask: the run's bounds, the diagonal, the window and the kept first keys --------
        const bool all_seen = kb >= klo && kb + kSpKeys - 1 <= khi && kb + kSpKeys - 1 <= wave_first
                              && (window == 0 || wave_last - kb < window || kb + kSpKeys - 1 < keep_first);
        if (!all_seen) {
            const int up = khi < qpos ? khi : qpos, low = (window > 0 && qpos - window + 1 > klo) ? qpos - window + 1 : klo;
#pragma unroll
            for (int tt = 0; tt < 2; ++tt)
#pragma unroll
                for (int r = 0; r < 16; ++r) {
                    const int key = kb + 32 * tt + 8 * (r >> 2) + 4 * half + (r & 3);
                    const bool seen = (key <= up) & ((key >= low) | ((key >= klo) & (key < keep_first)));
                    sacc[tt][r] = seen ? sacc[tt][r] : -INFINITY;
                }
        }
        // ---- running softmax, base 2: p = 2^(s c - m c) ---------------------------------
        float mloc = sacc[0][0];
#pragma unroll
        for (int tt = 0; tt < 2; ++tt)
#pragma unroll
            for (int r = 0; r < 16; ++r) mloc = fmaxf(mloc, sacc[tt][r]);
        mloc = fmaxf(mloc, __shfl_xor(mloc, 32, kWave));
        const float m_new = fmaxf(m, mloc);
        const float m_use = (m_new == -INFINITY) ? 0.f : m_new;
        const float mc = m_use * scale_log2e;
        const float corr = (m == -INFINITY) ? 0.f : __builtin_amdgcn_exp2f(m * scale_log2e - mc);
        float rs = 0.f;
#pragma unroll
        for (int tt = 0; tt < 2; ++tt)
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                const float p = __builtin_amdgcn_exp2f(fmaf(sacc[tt][r], scale_log2e, -mc));
                sacc[tt][r] = p;
                rs += p;
            }
        rs += __shfl_xor(rs, 32, kWave);
        l = l * corr + rs;
        m = m_new;
#pragma unroll
        for (int i = 0; i < ND; ++i)
#pragma unroll
            for (int r = 0; r < 16; ++r) oacc[i][r] *= corr;

        // ---- O^T += V^T P^T : four chunks of 16 keys ------------------------------------------
#pragma unroll
        for (int kc = 0; kc < 4; ++kc) {
            const int tt = kc >> 1, r0 = 8 * (kc & 1);
            sp_v8f pf;
#pragma unroll
            for (int e = 0; e < 8; ++e) pf[e] = sacc[tt][r0 + e];
            const sp_bf16x8 b = __builtin_convertvector(pf, sp_bf16x8);
#pragma unroll
            for (int dt = 0; dt < ND; ++dt) {
                const uint16_t* vp = Vs + (16 * kc + vrow) * PV + 32 * dt + vcol;
                const sp_v4s lo4 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((sp_v4s __attribute__((address_space(3)))*)vp);
                const sp_v4s hi4 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((sp_v4s __attribute__((address_space(3)))*)(vp + 8 * PV));
                const sp_bf16x8 a = __builtin_bit_cast(sp_bf16x8, __builtin_shufflevector(lo4, hi4, 0, 1, 2, 3, 4, 5, 6, 7));
                oacc[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, oacc[dt], 0, 0, 0);
            }
        }
    };
    if constexpr (ONE_STAGE) {
        for (int s = 0; s < n_steps; ++s) {
            __syncthreads();                               // the step before has been read
            stash(kreg0, vreg0, Ks0, Vs0);
            __syncthreads();
            if (s + 1 < n_steps) fetch(s + 1, kreg0, vreg0);
            if (s + 2 < n_steps) lookup(s + 2);
            compute(s, Ks0, Vs0);
        }
    } else
    for (int s = 0; s < n_steps; s += 2) {
        __syncthreads();                                   // stage 0 holds step s; stage 1 has been read
        if (s + 1 < n_steps) stash(kreg1, vreg1, Ks1, Vs1);
        if (s + 3 < n_steps) fetch(s + 3, kreg1, vreg1);
        if (s + 4 < n_steps) lookup(s + 4);
        compute(s, Ks0, Vs0);
        if (s + 1 >= n_steps) break;
        __syncthreads();                                   // stage 1 holds step s + 1; stage 0 has been read
        if (s + 2 < n_steps) stash(kreg0, vreg0, Ks0, Vs0);
        if (s + 4 < n_steps) fetch(s + 4, kreg0, vreg0);
        if (s + 5 < n_steps) lookup(s + 5);
        compute(s + 1, Ks1, Vs1);
    }

    if (!row_ok) return;
    if (sink) {                                            // exp(sink - m) joins the denominator
        const float sv = sinks ? sinks[h] * kLog2e : 0.f;
        const float mc = (m == -INFINITY) ? sv : m * scale_log2e;
        const float mf = fmaxf(mc, sv);
        const float corr = (m == -INFINITY) ? 0.f : __builtin_amdgcn_exp2f(mc - mf);
        l = l * corr + __builtin_amdgcn_exp2f(sv - mf);
#pragma unroll
        for (int i = 0; i < ND; ++i)
#pragma unroll
            for (int r = 0; r < 16; ++r) oacc[i][r] *= corr;
    }
    const float inv = 1.0f / l;
    uint16_t* op = out + (size_t)(row0 + my_row) * out_stride + (size_t)h * dv;
    const uint16_t* gp = gate ? gate + (size_t)(row0 + my_row) * gate_stride + (size_t)h * dv : nullptr;
#pragma unroll
    for (int dt = 0; dt < ND; ++dt)
#pragma unroll
        for (int r4 = 0; r4 < 4; ++r4) {
            const int d = 32 * dt + 8 * r4 + 4 * half;     // dims d .. d+3 are accumulators 4 r4 .. 4 r4 + 3
            if (MODE != kSpanPaged && d >= dv) continue;
            float o[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e] = oacc[dt][4 * r4 + e] * inv;
            if (gp) {
                const uint2 gv = *reinterpret_cast<const uint2*>(gp + d);
                o[0] *= sigmoid_f(__uint_as_float(gv.x << 16)); o[1] *= sigmoid_f(__uint_as_float(gv.x & 0xffff0000u));
                o[2] *= sigmoid_f(__uint_as_float(gv.y << 16)); o[3] *= sigmoid_f(__uint_as_float(gv.y & 0xffff0000u));
            }
            uint2 w;
            w.x = (uint32_t)f32_to_bf16_bits(o[0]) | ((uint32_t)f32_to_bf16_bits(o[1]) << 16);
            w.y = (uint32_t)f32_to_bf16_bits(o[2]) | ((uint32_t)f32_to_bf16_bits(o[3]) << 16);
            *reinterpret_cast<uint2*>(op + d) = w;
        }
}

