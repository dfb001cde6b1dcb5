// Attention through a latent: what is cached per token is ONE row [c | k_rot] of R + E values, shared by all
// heads: c (R values) is the normed latent that keys and values are made from, k_rot (E values) the rotated key
// part.  A head's key is W_uk c and its value W_uv c, so with q' = W_uk^T q_plain the score is
//     s = scale * (q' . c + q_rot . k_rot)
// and the head's result is W_uv (sum_j p_j c_j): the kernels here walk the latent rows only, every head against
// the same rows, and leave the two small products per head to the caller.
//
// Cache plane: [pages, 1, page_size, R + E].  Rotation: entries (2i, 2i+1) of the first `rot_dims` entries of a
// rotated part turn by the angle position * freq[i] (freq: float32 [2, rot_dims / 2], the frequency and what its rounding
// left) and are multiplied by rot_mult; the rest pass unchanged.  Angles, scores and the running softmax are float32.
// A query at position i sees key j when 0 <= i - j < window (window 0: every j <= i).  `sinks` (nullable, one float32 per
// head): exp(sinks[h]) joins the softmax's denominator, with no key and no value, not scaled.
//
// Prompt portions have two more ways: keys and values of every head made from the request's latent rows and walked by the
// matrix-core kernel of attn_span_prefill.h (ic_attn_latent_prefill), and two matrix products over the latent rows themselves
// with a masked softmax between them (ic_latent_gather, ic_latent_softmax).
#include "attn_span_prefill.h"
#include "rotation.h"

constexpr int kLatentMaxRank = 512;    // R: a lane holds R / 64 sums per head
constexpr int kLatentHeads = 4;        // heads that share one walk over the rows

// ---- per token: the query latent's norm, the key latent's norm, the rotated key part, the cache write -----------
// row[t] = [dq: Rq | dkv: R + E | ...].  cq[t] = rms(dq) * qn_w; cache[slot] = [rms(dkv[:R]) * kvn_w | rot(dkv[R:])].
template <typename T>
__global__ void __launch_bounds__(256)
latent_prep_kernel(const T* __restrict__ rows, int ld, int Rq, int R, int E, const float* __restrict__ qn_w,
                   const float* __restrict__ kvn_w, float eps, const float* __restrict__ freq, int rot_dims, float rot_mult,
                   const int* __restrict__ positions, T* __restrict__ cq, T* __restrict__ cache,
                   const int* __restrict__ slots) {
    __shared__ float red[8];
    const int t = blockIdx.x;
    const T* row = rows + (size_t)t * ld;
    float ss = 0.f;
    for (int j = threadIdx.x; j < Rq; j += blockDim.x) {
        const float v = to_f32(row[j]);
        ss += v * v;
    }
    float r = 1.0f / sqrtf(block_sum(ss, red) / (float)Rq + eps);
    for (int j = threadIdx.x; j < Rq; j += blockDim.x) cq[(size_t)t * Rq + j] = from_f32<T>(to_f32(row[j]) * r * qn_w[j]);
    if (!slots) return;
    const T* kv = row + Rq;
    T* dst = cache + (size_t)slots[t] * (R + E);
    ss = 0.f;
    for (int j = threadIdx.x; j < R; j += blockDim.x) {
        const float v = to_f32(kv[j]);
        ss += v * v;
    }
    r = 1.0f / sqrtf(block_sum(ss, red) / (float)R + eps);
    for (int j = threadIdx.x; j < R; j += blockDim.x) dst[j] = from_f32<T>(to_f32(kv[j]) * r * kvn_w[j]);
    const float pos = (float)positions[t];
    for (int i = threadIdx.x; i < rot_dims / 2; i += blockDim.x) {
        float c, s;
        pair_angle(pos, freq[i], freq[rot_dims / 2 + i], c, s);
        c *= rot_mult; s *= rot_mult;
        const float u = to_f32(kv[R + 2 * i]), v = to_f32(kv[R + 2 * i + 1]);
        dst[R + 2 * i] = from_f32<T>(u * c - v * s);
        dst[R + 2 * i + 1] = from_f32<T>(v * c + u * s);
    }
    for (int j = rot_dims + threadIdx.x; j < E; j += blockDim.x) dst[R + j] = kv[R + j];
}

IC_EXPORT int ic_latent_prep(const void* rows, int ld, int dtype, int Rq, int R, int E, const float* qn_w,
                             const float* kvn_w, float eps, const float* freq, int rot_dims, float rot_mult, const int* positions,
                             void* cq, void* cache, const int* slots, int T, hipStream_t stream) {
    if (T <= 0) return IC_OK;
    if (Rq <= 0 || R <= 0 || E < 0 || (slots && (!kvn_w || !cache)) || rot_dims < 0 || rot_dims > E || rot_dims % 2) return IC_ERR_ARG;
    if (dtype == IC_F32)
        hipLaunchKernelGGL(latent_prep_kernel<float>, dim3(T), dim3(256), 0, stream, (const float*)rows, ld, Rq, R, E, qn_w,
                           kvn_w, eps, freq, rot_dims, rot_mult, positions, (float*)cq, (float*)cache, slots);
    else if (dtype == IC_BF16)
        hipLaunchKernelGGL(latent_prep_kernel<bf16>, dim3(T), dim3(256), 0, stream, (const bf16*)rows, ld, Rq, R, E, qn_w,
                           kvn_w, eps, freq, rot_dims, rot_mult, positions, (bf16*)cq, (bf16*)cache, slots);
    else
        return IC_ERR_UNSUPPORTED;
    return ic_launch_status();
}

// ---- the queries' rotated parts: q[t, h, dim:dim+E] rotated into qa[t, h, R:R+E] (q itself with R = dim: a thread reads its
// entries before it writes them, and no two threads share one) ---------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256)
latent_q_rotate_kernel(const T* q, int q_stride, int dim, int E, int R, int H, const float* __restrict__ freq,
                       int rot_dims, float rot_mult, const int* __restrict__ positions, T* qa, int qa_stride) {
    const int t = blockIdx.x;
    const float pos = (float)positions[t];
    const int half = rot_dims / 2, rest = E - rot_dims, per = half + rest;
    for (int e = threadIdx.x; e < H * per; e += blockDim.x) {
        const int h = e / per, i = e % per;
        const T* src = q + (size_t)t * q_stride + (size_t)h * (dim + E) + dim;
        T* dst = qa + (size_t)t * qa_stride + (size_t)h * (R + E) + R;
        if (i < half) {
            float c, s;
            pair_angle(pos, freq[i], freq[half + i], c, s);
            c *= rot_mult; s *= rot_mult;
            const float u = to_f32(src[2 * i]), v = to_f32(src[2 * i + 1]);
            dst[2 * i] = from_f32<T>(u * c - v * s);
            dst[2 * i + 1] = from_f32<T>(v * c + u * s);
        } else {
            dst[rot_dims + i - half] = src[rot_dims + i - half];
        }
    }
}

IC_EXPORT int ic_latent_q_rotate(const void* q, int q_stride, int dtype, int dim, int E, int R, int H, const float* freq,
                                 int rot_dims, float rot_mult, const int* positions, void* qa, int qa_stride, int T, hipStream_t stream) {
    if (T <= 0 || E == 0) return IC_OK;
    if (dim < 0 || E < 0 || R <= 0 || H <= 0 || rot_dims < 0 || rot_dims > E || rot_dims % 2) return IC_ERR_ARG;
    if (dtype == IC_F32)
        hipLaunchKernelGGL(latent_q_rotate_kernel<float>, dim3(T), dim3(256), 0, stream, (const float*)q, q_stride, dim, E,
                           R, H, freq, rot_dims, rot_mult, positions, (float*)qa, qa_stride);
    else if (dtype == IC_BF16)
        hipLaunchKernelGGL(latent_q_rotate_kernel<bf16>, dim3(T), dim3(256), 0, stream, (const bf16*)q, q_stride, dim, E, R,
                           H, freq, rot_dims, rot_mult, positions, (bf16*)qa, qa_stride);
    else
        return IC_ERR_UNSUPPORTED;
    return ic_launch_status();
}

// ---- the walk over the latent rows ----------------------------------------------------------------------------------
// One wave per (token, group of up to kLatentHeads heads, split of the keys).  Scores: a lane owns one of 64 keys
// and reads its row in pieces of VEC values (16 bytes where the sizes allow), against the queries in LDS.
// Weighted sum: a lane owns pieces of the R columns and reads every key's row there.  With n_split > 1 each split
// leaves (max, sum, unnormalised row) in scratch memory and ic_attn_latent_merge finishes.
template <typename T, int VEC>
__global__ void __launch_bounds__(64)
attn_latent_kernel(const T* __restrict__ qa, int qa_stride, T* __restrict__ out, int out_stride,
                   const T* __restrict__ cache, const int* __restrict__ block_tables, int bt_stride,
                   const int* __restrict__ token_req, const int* __restrict__ positions,
                   const int* __restrict__ row_list, int H, int R, int E,
                   int page_size, float scale, int window, const float* __restrict__ sinks, int n_split,
                   float* __restrict__ part_acc, float* __restrict__ part_ml) {
    constexpr int HG = kLatentHeads, NP = kLatentMaxRank / 64 / VEC;   // pieces of VEC columns a lane owns
    extern __shared__ float qs[];                 // HG * (R + E) floats
    __shared__ float ps[HG][64];
    __shared__ long long krow[64];
    const int D = R + E, lane = threadIdx.x;
    const int n_groups = (H + HG - 1) / HG;
    const int hg = blockIdx.x % n_groups, split = blockIdx.y;
    const int t = row_list ? row_list[blockIdx.x / n_groups] : blockIdx.x / n_groups;
    const int h0 = hg * HG, nh = (H - h0 < HG) ? H - h0 : HG;
    const int pos = positions[t];
    const int* bt = block_tables + (size_t)token_req[t] * bt_stride;
    for (int e = lane; e < HG * D; e += 64) {
        const int g = e / D, d = e % D;
        qs[e] = g < nh ? to_f32(qa[(size_t)t * qa_stride + (size_t)(h0 + g) * D + d]) : 0.f;
    }
    __syncthreads();
    // this split's share of the keys lo..pos, in whole chunks of 64
    const int lo = (window > 0 && pos - window + 1 > 0) ? pos - window + 1 : 0;
    const int first_chunk = lo / 64, n_chunks = pos / 64 + 1 - first_chunk;
    const int per = (n_chunks + n_split - 1) / n_split;
    const int c_lo = first_chunk + split * per, c_hi = (split * per + per < n_chunks) ? c_lo + per : first_chunk + n_chunks;

    float acc[HG][NP][VEC];
#pragma unroll
    for (int g = 0; g < HG; ++g)
#pragma unroll
        for (int i = 0; i < NP; ++i)
#pragma unroll
            for (int v = 0; v < VEC; ++v) acc[g][i][v] = 0.f;
    float m[HG], l[HG];
#pragma unroll
    for (int g = 0; g < HG; ++g) { m[g] = -INFINITY; l[g] = 0.f; }

    for (int ch = c_lo; ch < c_hi; ++ch) {
        const int key = ch * 64 + lane;
        const bool valid = key >= lo && key <= pos;
        float s[HG];
#pragma unroll
        for (int g = 0; g < HG; ++g) s[g] = 0.f;
        long long base = 0;
        if (valid) {
            base = ((long long)bt[key / page_size] * page_size + key % page_size) * D;
            const T* kp = cache + base;
            for (int d = 0; d < D; d += VEC) {
                alignas(16) T kv[VEC];
                if (VEC == 1) kv[0] = kp[d];
                else *reinterpret_cast<uint4*>(kv) = *reinterpret_cast<const uint4*>(kp + d);
#pragma unroll
                for (int v = 0; v < VEC; ++v) {
                    const float kf = to_f32(kv[v]);
#pragma unroll
                    for (int g = 0; g < HG; ++g) s[g] += qs[g * D + d + v] * kf;
                }
            }
        }
        float corr[HG];
#pragma unroll
        for (int g = 0; g < HG; ++g) {
            const float sv = valid ? s[g] * scale : -INFINITY;
            const float m_new = fmaxf(m[g], wave_max(sv));      // finite: some key of every chunk is visible
            const float p = valid ? expf(sv - m_new) : 0.f;
            corr[g] = expf(m[g] - m_new);
            l[g] = l[g] * corr[g] + wave_sum(p);
            m[g] = m_new;
            ps[g][lane] = p;
        }
        krow[lane] = base;
        __syncthreads();
        const int k0 = (lo > ch * 64) ? lo - ch * 64 : 0, nk = (pos - ch * 64 + 1 < 64) ? pos - ch * 64 + 1 : 64;
#pragma unroll
        for (int g = 0; g < HG; ++g)
#pragma unroll
            for (int i = 0; i < NP; ++i)
#pragma unroll
                for (int v = 0; v < VEC; ++v) acc[g][i][v] *= corr[g];
        for (int kk = k0; kk < nk; ++kk) {
            const T* cp = cache + krow[kk];
            float pk[HG];
#pragma unroll
            for (int g = 0; g < HG; ++g) pk[g] = ps[g][kk];
#pragma unroll
            for (int i = 0; i < NP; ++i) {
                const int col = (lane + 64 * i) * VEC;
                if (col < R) {
                    alignas(16) T cv[VEC];
                    if (VEC == 1) cv[0] = cp[col];
                    else *reinterpret_cast<uint4*>(cv) = *reinterpret_cast<const uint4*>(cp + col);
#pragma unroll
                    for (int v = 0; v < VEC; ++v) {
                        const float cf = to_f32(cv[v]);
#pragma unroll
                        for (int g = 0; g < HG; ++g) acc[g][i][v] += pk[g] * cf;
                    }
                }
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int g = 0; g < HG; ++g) {
        if (g >= nh) continue;
        const int h = h0 + g;
        if (n_split == 1) {
            float inv = 1.0f / l[g];
            if (sinks) {
                const float mf = fmaxf(m[g], sinks[h]), c = expf(m[g] - mf);
                inv = c / (l[g] * c + expf(sinks[h] - mf));
            }
#pragma unroll
            for (int i = 0; i < NP; ++i) {
                const int col = (lane + 64 * i) * VEC;
                if (col < R) {
#pragma unroll
                    for (int v = 0; v < VEC; ++v)
                        out[(size_t)t * out_stride + (size_t)h * R + col + v] = from_f32<T>(acc[g][i][v] * inv);
                }
            }
        } else {
            const size_t pi = ((size_t)t * H + h) * n_split + split;
            if (lane == 0) { part_ml[2 * pi] = m[g]; part_ml[2 * pi + 1] = l[g]; }
#pragma unroll
            for (int i = 0; i < NP; ++i) {
                const int col = (lane + 64 * i) * VEC;
                if (col < R) {
#pragma unroll
                    for (int v = 0; v < VEC; ++v) part_acc[pi * R + col + v] = acc[g][i][v];
                }
            }
        }
    }
}

// ---- the same walk on the matrix cores (bfloat16) --------------------------------------------------------------------
// One block per (token, group of up to 32 heads, split of the keys); the heads are the 32 "queries" of
// v_mfma_f32_32x32x16_bf16.  A step of 32 keys is loaded once into LDS as padded rows.  Scores are computed
// transposed, S^T = K Q^T (A = 32 key rows x 16 values out of LDS, B = the heads' queries, held in registers), so a
// lane holds 16 keys of ONE head, its partner lane (l ^ 32) the other 16, and the probabilities are already the B
// operand of O^T = V^T P^T, whose A operand (the first R values of the same LDS rows, transposed) comes out of LDS
// through the transposing read.  Operand layout (lane l, h = l / 32): A[i = l % 32][k = 8h..8h+7],
// B[k = 8h..8h+7][j = l % 32], D[i = 8(r / 4) + 4h + r % 4][j = l % 32] for the 16 accumulators r.
// A key outside the token's window or beyond its position is replaced by the nearest one inside when loaded, and masked.
typedef __bf16 lat_bf16x8 __attribute__((ext_vector_type(8)));
typedef float lat_v16f __attribute__((ext_vector_type(16)));
typedef float lat_v8f __attribute__((ext_vector_type(8)));
typedef short lat_v4s __attribute__((ext_vector_type(4)));

template <int R, int E>
__global__ void __launch_bounds__(64 * (R >= 128 ? 4 : R / 32))
attn_latent_mfma_kernel(const bf16* __restrict__ qa, int qa_stride, bf16* __restrict__ out, int out_stride,
                        const bf16* __restrict__ cache, const int* __restrict__ block_tables, int bt_stride,
                        const int* __restrict__ token_req, const int* __restrict__ positions,
                        const int* __restrict__ row_list, int H, int page_size, float scale, int window,
                        const float* __restrict__ sinks, int n_split, float* __restrict__ part_acc,
                        float* __restrict__ part_ml) {
    // The block's waves share a step's rows in LDS; each computes the (same) scores and owns ND / WAVES of the
    // 32-column tiles of the result.
    constexpr int D = R + E, NC = D / 16, ND = R / 32, PK = D + 8, PIECES = D / 8;
    constexpr int WAVES = ND >= 4 ? 4 : ND, NDW = ND / WAVES, THREADS = 64 * WAVES;
    constexpr int TPR = THREADS / 32, NL = (PIECES + TPR - 1) / TPR; // threads that load a row, 16-byte pieces each of them loads
    constexpr bool QLDS = NC > 20;         // long rows: the queries wait in LDS (in registers they would halve the waves a unit holds)
    __shared__ __attribute__((aligned(16))) uint16_t Ks[32 * PK];
    __shared__ __attribute__((aligned(16))) uint16_t Qs[QLDS ? 32 * PK : 8];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lq = lane & 31, half = lane >> 5;
    const int n_groups = (H + 31) / 32;
    const int hg = blockIdx.x % n_groups, split = blockIdx.y;
    const int t = row_list ? row_list[blockIdx.x / n_groups] : blockIdx.x / n_groups;
    const int head = hg * 32 + lq;
    const bool row_ok = head < H;
    const int pos = positions[t];
    const int* bt = block_tables + (size_t)token_req[t] * bt_stride;

    lat_bf16x8 qf[QLDS ? 1 : NC];
    {
        const bf16* qp = qa + (size_t)t * qa_stride + (size_t)(row_ok ? head : 0) * D + 8 * half;
#pragma unroll
        for (int c = 0; c < NC; ++c) {
            if (QLDS && c % WAVES != wave) continue;          // the waves write the queries' pieces in turn
            uint4 v = *reinterpret_cast<const uint4*>(qp + 16 * c);
            if (!row_ok) v = uint4{0u, 0u, 0u, 0u};
            if (QLDS) *reinterpret_cast<uint4*>(Qs + lq * PK + 16 * c + 8 * half) = v;
            else qf[c] = __builtin_bit_cast(lat_bf16x8, v);
        }
    }
    const int lo = (window > 0 && pos - window + 1 > 0) ? pos - window + 1 : 0;
    const int first_step = lo / 32, n_steps = pos / 32 + 1 - first_step;
    const int per = (n_steps + n_split - 1) / n_split;
    const int s_lo = first_step + split * per, s_hi = (split * per + per < n_steps) ? s_lo + per : first_step + n_steps;

    lat_v16f oacc[NDW];
#pragma unroll
    for (int i = 0; i < NDW; ++i)
#pragma unroll
        for (int r = 0; r < 16; ++r) oacc[i][r] = 0.f;
    float m = -INFINITY, l = 0.f;
    const float scale_log2e = scale * 1.4426950408889634f;
    const int vrow = 4 * half + ((lane & 15) >> 2);
    const int vcol = 16 * ((lane >> 4) & 1) + 4 * (lane & 3);

    // A step's rows are asked for one step ahead: while this step is computed out of LDS the next one's loads are in flight.
    // (TPR threads share a row, so a thread looks up one page a step.)
    const int my_row = threadIdx.x / TPR, my_piece = threadIdx.x % TPR;
    sp_v4u got[NL];
    auto fetch = [&](int step) {
        const int want = 32 * step + my_row;
        const int key = (want < lo) ? lo : (want < pos) ? want : pos;
        const bf16* src = cache + ((long long)bt[key / page_size] * page_size + key % page_size) * D + my_piece * 8;
#pragma unroll
        for (int k = 0; k < NL; ++k) {
            if (PIECES % TPR == 0 || my_piece + TPR * k < PIECES) got[k] = *reinterpret_cast<const sp_v4u*>(src + TPR * 8 * k);
            else got[k] = sp_v4u{0u, 0u, 0u, 0u};
        }
    };
    if (s_lo < s_hi) fetch(s_lo);
    for (int s = s_lo; s < s_hi; ++s) {
        const int kb = 32 * s;
#pragma unroll
        for (int k = 0; k < NL; ++k)
            if (PIECES % TPR == 0 || my_piece + TPR * k < PIECES) *reinterpret_cast<sp_v4u*>(Ks + my_row * PK + (my_piece + TPR * k) * 8) = got[k];
        __syncthreads();
        if (s + 1 < s_hi) fetch(s + 1);
        lat_v16f sacc, sacc2;                  // two chains of dependent products instead of one
#pragma unroll
        for (int r = 0; r < 16; ++r) sacc[r] = sacc2[r] = 0.f;
#pragma unroll
        for (int c = 0; c < NC; ++c) {
            const lat_bf16x8 a = *reinterpret_cast<const lat_bf16x8*>(Ks + lq * PK + 16 * c + 8 * half);
            const lat_bf16x8 q = QLDS ? *reinterpret_cast<const lat_bf16x8*>(Qs + lq * PK + 16 * c + 8 * half) : qf[c];
            if (c & 1) sacc2 = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, q, sacc2, 0, 0, 0);
            else sacc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, q, sacc, 0, 0, 0);
        }
#pragma unroll
        for (int r = 0; r < 16; ++r) sacc[r] += sacc2[r];
        if (kb + 31 > pos || kb < lo) {
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                const int key = kb + 8 * (r >> 2) + 4 * half + (r & 3);
                if (key > pos || key < lo) sacc[r] = -INFINITY;
            }
        }
        float mloc = sacc[0];
#pragma unroll
        for (int r = 1; r < 16; ++r) mloc = fmaxf(mloc, sacc[r]);
        mloc = fmaxf(mloc, __shfl_xor(mloc, 32, kWave));
        const float m_new = fmaxf(m, mloc);                     // finite: some key of every step is visible
        const float mc = m_new * scale_log2e;
        const float corr = (m == -INFINITY) ? 0.f : __builtin_amdgcn_exp2f(m * scale_log2e - mc);
        float rs = 0.f;
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const float p = __builtin_amdgcn_exp2f(fmaf(sacc[r], scale_log2e, -mc));
            sacc[r] = p;
            rs += p;
        }
        rs += __shfl_xor(rs, 32, kWave);
        l = l * corr + rs;
        m = m_new;
#pragma unroll
        for (int i = 0; i < NDW; ++i)
#pragma unroll
            for (int r = 0; r < 16; ++r) oacc[i][r] *= corr;
#pragma unroll
        for (int kc = 0; kc < 2; ++kc) {
            lat_v8f pf;
#pragma unroll
            for (int e = 0; e < 8; ++e) pf[e] = sacc[8 * kc + e];
            const lat_bf16x8 b = __builtin_convertvector(pf, lat_bf16x8);
#pragma unroll
            for (int dt = 0; dt < NDW; ++dt) {
                const uint16_t* vp = Ks + (16 * kc + vrow) * PK + 32 * (wave * NDW + dt) + vcol;
                const lat_v4s lo4 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lat_v4s __attribute__((address_space(3)))*)vp);
                const lat_v4s hi4 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lat_v4s __attribute__((address_space(3)))*)(vp + 8 * PK));
                const lat_bf16x8 a = __builtin_bit_cast(lat_bf16x8, __builtin_shufflevector(lo4, hi4, 0, 1, 2, 3, 4, 5, 6, 7));
                oacc[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, oacc[dt], 0, 0, 0);
            }
        }
        __syncthreads();
    }
    if (!row_ok) return;
    if (n_split == 1) {
        float inv = 1.0f / l;
        if (sinks) {                              // the term exp(sink) joins the denominator (exponents base 2)
            const float sv = sinks[head] * kLog2e, ms = m * scale_log2e, mf = fmaxf(ms, sv), c = __builtin_amdgcn_exp2f(ms - mf);
            inv = c / (l * c + __builtin_amdgcn_exp2f(sv - mf));
        }
        bf16* op = out + (size_t)t * out_stride + (size_t)head * R + 32 * wave * NDW;
#pragma unroll
        for (int dt = 0; dt < NDW; ++dt)
#pragma unroll
            for (int r = 0; r < 16; ++r) op[32 * dt + 8 * (r >> 2) + 4 * half + (r & 3)] = __float2bfloat16(oacc[dt][r] * inv);
    } else {
        const size_t pi = ((size_t)t * H + head) * n_split + split;
        if (half == 0 && wave == 0) { part_ml[2 * pi] = m * scale; part_ml[2 * pi + 1] = l; }
#pragma unroll
        for (int dt = 0; dt < NDW; ++dt)
#pragma unroll
            for (int r = 0; r < 16; ++r)
                part_acc[pi * R + 32 * (wave * NDW + dt) + 8 * (r >> 2) + 4 * half + (r & 3)] = oacc[dt][r];
    }
}

template <int R, int E>
static void latent_mfma_launch(dim3 grid, hipStream_t stream, const void* qa, int qa_stride, void* out, int out_stride,
                               const void* cache, const int* block_tables, int bt_stride, const int* token_req,
                               const int* positions, const int* row_list, int H, int page_size, float scale, int window,
                               const float* sinks, int n_split, float* part_acc, float* part_ml) {
    hipLaunchKernelGGL((attn_latent_mfma_kernel<R, E>), grid, dim3(64 * (R >= 128 ? 4 : R / 32)), 0, stream, (const bf16*)qa, qa_stride, (bf16*)out,
                       out_stride, (const bf16*)cache, block_tables, bt_stride, token_req, positions, row_list, H, page_size,
                       scale, window, sinks, n_split, part_acc, part_ml);
}

// Sizes the matrix-core walk is built for: the latent 64, 128, 256 or 512 wide, the rotated part 16, 32 or 64.
IC_EXPORT int ic_attn_latent_on_matrix_cores(int dtype, int R, int E) {
    return dtype == IC_BF16 && (R == 64 || R == 128 || R == 256 || R == 512) && (E == 16 || E == 32 || E == 64);
}

// Merge of the splits: one block per (token, head).
template <typename T>
__global__ void __launch_bounds__(256)
attn_latent_merge_kernel(const float* __restrict__ part_acc, const float* __restrict__ part_ml, int n_split, int H, int R,
                         T* __restrict__ out, int out_stride, const int* __restrict__ row_list, const float* __restrict__ sinks) {
    const int h = blockIdx.x % H, t = row_list ? row_list[blockIdx.x / H] : blockIdx.x / H;
    const size_t p0 = ((size_t)t * H + h) * n_split;
    __shared__ float wgt[64];                 // a split's share of the result: exp(m_s - m) / l
    if (threadIdx.x < 64) {
        const int sp = threadIdx.x;
        const float ms = sp < n_split ? part_ml[2 * (p0 + sp)] : -INFINITY;
        const float ls = sp < n_split ? part_ml[2 * (p0 + sp) + 1] : 0.f;
        float m = wave_max(ms);
        if (sinks) m = fmaxf(m, sinks[h]);
        const float e = ms > -INFINITY ? expf(ms - m) : 0.f;
        const float l = wave_sum(ls * e) + (sinks ? expf(sinks[h] - m) : 0.f);
        wgt[sp] = e / l;
    }
    __syncthreads();
    for (int j = threadIdx.x; j < R; j += blockDim.x) {
        float a = 0.f;
#pragma unroll 4
        for (int sp = 0; sp < n_split; ++sp) a += part_acc[(p0 + sp) * R + j] * wgt[sp];     // (an empty split left zeros)
        out[(size_t)t * out_stride + (size_t)h * R + j] = from_f32<T>(a);
    }
}

IC_EXPORT int ic_attn_latent(const void* qa, int qa_stride, void* out, int out_stride, int dtype, const void* cache,
                             const int* block_tables, int bt_stride, const int* token_req, const int* positions,
                             const int* row_list, int T, int H, int R, int E, int page_size, float scale, int window,
                             const float* sinks, int n_split,
                             float* part_acc, float* part_ml, int force_vector, hipStream_t stream) {
    if (T <= 0) return IC_OK;
    if (H <= 0 || R <= 0 || R > kLatentMaxRank || E < 0 || page_size <= 0 || window < 0 || n_split < 1 || n_split > 64) return IC_ERR_ARG;
    if (n_split > 1 && (!part_acc || !part_ml)) return IC_ERR_ARG;
    const int D = R + E;
    const size_t lds = (size_t)kLatentHeads * D * sizeof(float);
    if (lds > 60 * 1024) return IC_ERR_TOO_LARGE;
    if (ic_attn_latent_on_matrix_cores(dtype, R, E) && scale > 0.f && !force_vector) {
        const int wide_groups = (H + 31) / 32;
        if ((long long)T * wide_groups > 0x7fffffffLL) return IC_ERR_ARG;
        dim3 wide((unsigned)(T * wide_groups), n_split);
#define IC_LATM(RR, EE)                                                                                                  \
    if (R == RR && E == EE)                                                                                              \
        latent_mfma_launch<RR, EE>(wide, stream, qa, qa_stride, out, out_stride, cache, block_tables, bt_stride, token_req, \
                                   positions, row_list, H, page_size, scale, window, sinks, n_split, part_acc, part_ml);
        IC_LATM(64, 16) IC_LATM(64, 32) IC_LATM(64, 64) IC_LATM(128, 16) IC_LATM(128, 32) IC_LATM(128, 64)
        IC_LATM(256, 16) IC_LATM(256, 32) IC_LATM(256, 64) IC_LATM(512, 16) IC_LATM(512, 32) IC_LATM(512, 64)
#undef IC_LATM
        if (n_split > 1)
            hipLaunchKernelGGL(attn_latent_merge_kernel<bf16>, dim3(T * H), dim3(256), 0, stream, part_acc, part_ml, n_split, H,
                               R, (bf16*)out, out_stride, row_list, sinks);
        return ic_launch_status();
    }
    const int n_groups = (H + kLatentHeads - 1) / kLatentHeads;
    if ((long long)T * n_groups > 0x7fffffffLL) return IC_ERR_ARG;
    dim3 grid((unsigned)(T * n_groups), n_split), block(64);
#define IC_LAT(TT, VV)                                                                                                 \
    hipLaunchKernelGGL((attn_latent_kernel<TT, VV>), grid, block, lds, stream, (const TT*)qa, qa_stride, (TT*)out,     \
                       out_stride, (const TT*)cache, block_tables, bt_stride, token_req, positions, row_list, H, R, E,  \
                       page_size, scale, window, sinks, n_split, part_acc, part_ml)
    if (dtype == IC_F32) {
        if (R % 4 == 0 && E % 4 == 0) IC_LAT(float, 4); else IC_LAT(float, 1);
    } else if (dtype == IC_BF16) {
        if (R % 8 == 0 && E % 8 == 0) IC_LAT(bf16, 8); else IC_LAT(bf16, 1);
    } else
        return IC_ERR_UNSUPPORTED;
#undef IC_LAT
    if (n_split > 1) {
        if (dtype == IC_F32)
            hipLaunchKernelGGL(attn_latent_merge_kernel<float>, dim3(T * H), dim3(256), 0, stream, part_acc, part_ml, n_split,
                               H, R, (float*)out, out_stride, row_list, sinks);
        else
            hipLaunchKernelGGL(attn_latent_merge_kernel<bf16>, dim3(T * H), dim3(256), 0, stream, part_acc, part_ml, n_split,
                               H, R, (bf16*)out, out_stride, row_list, sinks);
    }
    return ic_launch_status();
}

// ---- prompt portions: keys and values made per head --------------------------------------------------------------------
// `kv` holds one row per key from key0 on, every head's key part and, from column v_off on, every head's value (a product of
// the gathered latent rows); `rows` the gathered rows themselves, whose last E columns are the shared rotated key part.  The
// portion's tokens are rows row0 .. row0 + n - 1 of q (rotated in place), out and gate, at positions pos0 and up.
// Key sizes dim + E up to 192 and values up to 128, each made of whole 16-byte pieces.
IC_EXPORT int ic_attn_latent_prefill_supported(int dtype, int dim, int E, int dv) {
    return dtype == IC_BF16 && dim > 0 && E >= 0 && dv > 0 && dim % 8 == 0 && E % 8 == 0 && dv % 8 == 0 && dim + E <= 192 && dv <= 128;
}

IC_EXPORT int ic_attn_latent_prefill(const void* q, int q_stride, void* out, int out_stride, const void* gate, int gate_stride, int dtype,
                                     const void* kv, int kv_stride, int v_off, const void* rows, int rows_stride, int R, int key0,
                                     int row0, int n, int pos0, int H, int dim, int E, int dv, float scale, int window,
                                     const float* sinks, hipStream_t stream) {
    if (n <= 0) return IC_OK;
    if (!ic_attn_latent_prefill_supported(dtype, dim, E, dv)) return IC_ERR_UNSUPPORTED;
    const int first = (window > 0 && pos0 - window + 1 > 0) ? pos0 - window + 1 : 0;
    if (H <= 0 || R < 0 || window < 0 || row0 < 0 || pos0 < 0 || key0 < 0 || key0 > first || !(scale > 0.f)) return IC_ERR_ARG;
    const uint16_t* krot = (const uint16_t*)rows + R;
    if ((q_stride | kv_stride | v_off | rows_stride) & 7 || (out_stride & 3) || (gate && (gate_stride & 3)) ||
        ((uintptr_t)q & 15) || ((uintptr_t)kv & 15) || ((uintptr_t)krot & 15) || ((uintptr_t)out & 7) || ((uintptr_t)gate & 7))
        return IC_ERR_ARG;
    const long long blocks = (long long)((n + kSpRows - 1) / kSpRows) * H;
    if (blocks > 0x7fffffffLL) return IC_ERR_ARG;
    const SpanSizes z{dim + E, dv, E, kv_stride, v_off, key0, rows_stride, krot, int4{0, row0, n, pos0}};
    const int dk = dim + E;
#define IC_LATP(K, V)                                                                                                        \
    if (dk <= K && dv <= V) {                                                                                                \
        hipLaunchKernelGGL((attn_span_prefill_kernel<K, V, kSpanLatent>), dim3((unsigned)blocks), dim3(256), 0, stream,       \
                           (const uint16_t*)q, q_stride, (uint16_t*)out, out_stride, (const uint16_t*)gate, gate_stride,      \
                           (const uint16_t*)kv, nullptr, nullptr, 0, nullptr, H, H, 0, scale * kLog2e, window, 0,             \
                           sinks ? 1 : 0, sinks, 0.f, nullptr, z);                                                           \
        return ic_launch_status();                                                                                           \
    }
    IC_LATP(64, 64) IC_LATP(64, 96) IC_LATP(96, 64) IC_LATP(96, 96) IC_LATP(128, 64) IC_LATP(128, 128) IC_LATP(192, 64) IC_LATP(192, 128)
#undef IC_LATP
    return IC_ERR_UNSUPPORTED;
}

// ---- prompt portions through matrix products -------------------------------------------------------------------------
// For a portion of several tokens the walk is two products over all heads at once, rows = (token, head):
// scores = Q' C^T and result = P C[:, :R].  The request's latent rows are gathered out of their pages into one
// matrix (and its first R columns transposed, for the second product), the scores pass a masked softmax.

// Row j of `rows` is key key0 + j.  rows[j] = the cache row of its key for first <= key < L, zeros for the other keys up to
// L_pad rows; rows_t[c, j] = rows[j, c] for c < R (rows_t null: left out).
template <typename T>
__global__ void __launch_bounds__(256)
latent_gather_kernel(const T* __restrict__ cache, const int* __restrict__ table, int page_size, int D, int R, int key0, int first,
                     int L, int L_pad, T* __restrict__ rows, T* __restrict__ rows_t) {
    // blockIdx.y == 0: 64 keys' rows as they are; blockIdx.y = 1 + i: columns 64 i .. 64 i + 63 of the same keys, transposed
    __shared__ T tile[64][65];
    const int j0 = blockIdx.x * 64, lane = threadIdx.x % 64, w = threadIdx.x / 64;
    if (blockIdx.y == 0) {
        for (int jj = w; jj < 64; jj += 4) {
            const int j = j0 + jj, key = key0 + j;
            if (j >= L_pad) break;
            const T* src = (key >= first && key < L) ? cache + ((long long)table[key / page_size] * page_size + key % page_size) * D : nullptr;
            for (int c = lane; c < D; c += 64) rows[(size_t)j * D + c] = src ? src[c] : from_f32<T>(0.f);
        }
        return;
    }
    const int c0 = 64 * (blockIdx.y - 1);
    for (int jj = w; jj < 64; jj += 4) {
        const int j = j0 + jj, key = key0 + j, c = c0 + lane;
        T v = from_f32<T>(0.f);
        if (j < L_pad && key >= first && key < L && c < R) v = cache[((long long)table[key / page_size] * page_size + key % page_size) * D + c];
        tile[jj][lane] = v;
    }
    __syncthreads();
    for (int cc = w; cc < 64; cc += 4) {
        const int c = c0 + cc, j = j0 + lane;
        if (c < R && j < L_pad) rows_t[(size_t)c * L_pad + j] = tile[lane][cc];
    }
}

// The rows alone, 16 bytes a thread (rows and cache of whole 16-byte pieces).
__global__ void __launch_bounds__(256)
latent_gather_vec_kernel(const uint4* __restrict__ cache, const int* __restrict__ table, int page_size, int pieces, int key0, int first,
                         int L, int L_pad, uint4* __restrict__ rows) {
    const long long e = (long long)blockIdx.x * 256 + threadIdx.x;
    const int j = (int)(e / pieces), c = (int)(e % pieces), key = key0 + j;
    if (j >= L_pad) return;
    uint4 v = uint4{0u, 0u, 0u, 0u};
    if (key >= first && key < L) v = cache[((long long)table[key / page_size] * page_size + key % page_size) * pieces + c];
    rows[e] = v;
}

IC_EXPORT int ic_latent_gather(const void* cache, int dtype, const int* table, int page_size, int D, int R, int key0, int first, int L,
                               int L_pad, void* rows, void* rows_t, hipStream_t stream) {
    if (L <= 0) return IC_OK;
    if (page_size <= 0 || D <= 0 || R <= 0 || R > D || key0 < 0 || first < key0 || L <= first || L_pad < L - key0) return IC_ERR_ARG;
    const int piece = dtype == IC_F32 ? 4 : 8;
    if (!rows_t && (dtype == IC_F32 || dtype == IC_BF16) && D % piece == 0 && (((uintptr_t)cache | (uintptr_t)rows) & 15) == 0) {
        const long long blocks = ((long long)L_pad * (D / piece) + 255) / 256;
        if (blocks > 0x7fffffffLL) return IC_ERR_TOO_LARGE;
        hipLaunchKernelGGL(latent_gather_vec_kernel, dim3((unsigned)blocks), dim3(256), 0, stream, (const uint4*)cache, table, page_size,
                           D / piece, key0, first, L, L_pad, (uint4*)rows);
        return ic_launch_status();
    }
    dim3 grid((L_pad + 63) / 64, rows_t ? 1 + (R + 63) / 64 : 1), block(256);
    if (dtype == IC_F32)
        hipLaunchKernelGGL(latent_gather_kernel<float>, grid, block, 0, stream, (const float*)cache, table, page_size, D, R, key0, first,
                           L, L_pad, (float*)rows, (float*)rows_t);
    else if (dtype == IC_BF16)
        hipLaunchKernelGGL(latent_gather_kernel<bf16>, grid, block, 0, stream, (const bf16*)cache, table, page_size, D, R, key0, first,
                           L, L_pad, (bf16*)rows, (bf16*)rows_t);
    else
        return IC_ERR_UNSUPPORTED;
    return ic_launch_status();
}

// Column j of a row is key key0 + j.  Row m belongs to token m / H of the portion, at position pos0 + m / H, and head m % H;
// p = softmax(scale * s) over the keys it sees (window, sinks: see above), zero elsewhere.  One block per row; the scores are
// float32.
template <typename T>
__global__ void __launch_bounds__(256)
latent_softmax_kernel(const float* __restrict__ s, int lds, T* __restrict__ p, int ldp, int H, int n_cols, int key0, int pos0,
                      float scale, int window, const float* __restrict__ sinks) {
    __shared__ float red[8];
    const int m = blockIdx.x, pos = pos0 + m / H;
    const int n = min(pos - key0 + 1, n_cols);                       // columns lo .. n - 1 are seen
    const int lo = window > 0 ? max(pos - window + 1 - key0, 0) : 0;
    const float* row = s + (size_t)m * lds;
    T* out = p + (size_t)m * ldp;
    const float sink = sinks ? sinks[m % H] : -INFINITY;
    if (n_cols <= 16 * 256) {                 // the row is read once and waits in registers
        float v[16];
        float mx = -INFINITY;
#pragma unroll
        for (int k = 0; k < 16; ++k) {
            const int j = threadIdx.x + 256 * k;
            v[k] = (j >= lo && j < n) ? row[j] : -INFINITY;
            mx = fmaxf(mx, v[k]);
        }
        mx = fmaxf(block_max(mx, red) * scale, sink);
        float sum = 0.f;
#pragma unroll
        for (int k = 0; k < 16; ++k) {
            v[k] = expf(v[k] * scale - mx);       // exp(-inf) = 0 for the keys that are not seen
            sum += v[k];
        }
        sum = block_sum(sum, red);
        const float inv = 1.0f / (sum + (sinks ? expf(sink - mx) : 0.f));
#pragma unroll
        for (int k = 0; k < 16; ++k) {
            const int j = threadIdx.x + 256 * k;
            if (j < n_cols) out[j] = from_f32<T>(v[k] * inv);
        }
        return;
    }
    float mx = -INFINITY;
    for (int j = lo + threadIdx.x; j < n; j += blockDim.x) mx = fmaxf(mx, row[j]);
    mx = fmaxf(block_max(mx, red) * scale, sink);
    float sum = 0.f;
    for (int j = lo + threadIdx.x; j < n; j += blockDim.x) sum += expf(row[j] * scale - mx);
    sum = block_sum(sum, red);
    const float inv = 1.0f / (sum + (sinks ? expf(sink - mx) : 0.f));
    for (int j = threadIdx.x; j < n_cols; j += blockDim.x)
        out[j] = from_f32<T>((j >= lo && j < n) ? expf(row[j] * scale - mx) * inv : 0.f);
}

IC_EXPORT int ic_latent_softmax(const float* s, int lds, void* p, int ldp, int dtype, int M, int H, int n_cols, int key0, int pos0,
                                float scale, int window, const float* sinks, hipStream_t stream) {
    if (M <= 0) return IC_OK;
    if (H <= 0 || n_cols <= 0 || pos0 < key0 || key0 < 0 || window < 0 || scale <= 0.f) return IC_ERR_ARG;
    if (dtype == IC_F32)
        hipLaunchKernelGGL(latent_softmax_kernel<float>, dim3(M), dim3(256), 0, stream, s, lds, (float*)p, ldp, H, n_cols, key0,
                           pos0, scale, window, sinks);
    else if (dtype == IC_BF16)
        hipLaunchKernelGGL(latent_softmax_kernel<bf16>, dim3(M), dim3(256), 0, stream, s, lds, (bf16*)p, ldp, H, n_cols, key0,
                           pos0, scale, window, sinks);
    else
        return IC_ERR_UNSUPPORTED;
    return ic_launch_status();
}
